// Whole prompts of attention through a latent, as attention with keys and values a head (bfloat16, matrix cores):
// the step's latents have been multiplied with every head's key and value matrices, and what is here puts queries,
// keys and values where the prompt kernel of attention_mfma.h reads them, and runs it for the widths that come up
// (keys of dim + rot dimensions, values of another width), with a window or with a sink and a gate.
#include "attention_mfma.h"
#include <algorithm>

// Eight neighbouring dimensions d0 .. d0 + 7 of a part of `rot` floats whose first rot_dims are rotated in pairs
// (pairing 0: i with i + rot_dims / 2; 1: neighbours) by the token's table row, as bfloat16.
__device__ __forceinline__ uint4 rotated_oct(const float* __restrict__ part, int d0, int rot, int rot_dims, int pairing,
                                             const float2* __restrict__ tab) {
    float v[8];
    const int half = rot_dims / 2;
#pragma unroll
    for (int e = 0; e < 8; ++e) {
        const int i = d0 + e;
        v[e] = 0.f;
        if (i < rot) {
            v[e] = part[i];
            if (i < rot_dims) {
                const bool second = pairing ? (i & 1) : i >= half;
                const float2 c = tab[pairing ? i >> 1 : (second ? i - half : i)];
                const float other = part[pairing ? i ^ 1 : (second ? i - half : i + half)];
                v[e] = second ? fmaf(v[e], c.x, other * c.y) : fmaf(v[e], c.x, -other * c.y);
            }
        }
    }
    return make_uint4(pack_bf16(v[0], v[1]), pack_bf16(v[2], v[3]), pack_bf16(v[4], v[5]), pack_bf16(v[6], v[7]));
}

// One block a (page of 64 tokens, head).  kvh bfloat16 [T, H * (dim + dv)]: every head's unrotated keys [H][dim], then every
// head's values [H][dv]; kv float [T, ldkv]: from `rank` on the shared rotated key part, not yet rotated; q float
// [T, ldq]: per head [dim | rot].  Writes q_out [T][H][dim + rot] and the head's part of the step's own pages: keys
// [dim | rotated part], values.  dim, rot and dv are multiples of 8, dv of 16.  Rows of tokens that are not there are not written.
__global__ __launch_bounds__(256) void latent_heads_kernel(const bf16_t* __restrict__ kvh, const float* __restrict__ kv, int ldkv, int rank,
                                                           const float* __restrict__ q, int ldq, const float2* __restrict__ cs,
                                                           bf16_t* __restrict__ q_out, bf16_t* __restrict__ k_pool,
                                                           bf16_t* __restrict__ v_pool, const int* __restrict__ table, int table_stride,
                                                           const int* __restrict__ cu, int batch, int H, int dim, int rot, int rot_dims,
                                                           int pairing, int dv) {
    const int h = blockIdx.y, tid = threadIdx.x;
    int page = blockIdx.x, b = 0, first = 0, n = 0;
    for (; b < batch; ++b) {
        const int len = cu[b + 1] - cu[b], pages = (len + kPageTokens - 1) / kPageTokens;
        if (page < pages) { first = cu[b] + page * kPageTokens; n = min(kPageTokens, cu[b + 1] - first); break; }
        page -= pages;
    }
    if (b >= batch) return;
    const int dk = dim + rot, octs = dk / 8, half = rot_dims / 2;
    const size_t at = (size_t)table[(size_t)b * table_stride + page] * H + h;
    bf16_t* kp = k_pool + at * kPageTokens * dk;
    bf16_t* vp = v_pool + at * kPageTokens * dv;
    const size_t ld = (size_t)H * (dim + dv);
    // keys: piece e of the page is 8 dimensions of one token (common.h: page_key_offset), in the order they lie there
    for (int e = tid; e < kPageTokens * octs; e += 256) {
        const int i = e & 15, o = (e >> 4) % octs, rb = (e >> 4) / octs;
        const int tok = 16 * (i >> 2) + 4 * rb + (i & 3), d0 = 8 * o;
        if (tok >= n) continue;
        const int t = first + tok;
        *reinterpret_cast<uint4*>(kp + (size_t)e * 8) =
            d0 < dim ? *reinterpret_cast<const uint4*>(kvh + t * ld + (size_t)h * dim + d0)
                     : rotated_oct(kv + (size_t)t * ldkv + rank, d0 - dim, rot, rot_dims, pairing, cs + (size_t)t * half);
    }
    // values: piece e is 8 tokens of one dimension (page_value_offset)
    for (int e = tid; e < dv * 8; e += 256) {
        const int d = 16 * (e >> 7) + (e & 15), tok0 = 16 * ((e >> 4) & 3) + 8 * ((e >> 6) & 1);
        if (tok0 >= n) continue;
        uint32_t u[8];
#pragma unroll
        for (int j = 0; j < 8; ++j) u[j] = tok0 + j < n ? kvh[(first + tok0 + j) * ld + (size_t)H * dim + (size_t)h * dv + d] : 0u;
        *reinterpret_cast<uint4*>(vp + (size_t)e * 8) = make_uint4(u[0] | (u[1] << 16), u[2] | (u[3] << 16), u[4] | (u[5] << 16), u[6] | (u[7] << 16));
    }
    // queries
    for (int e = tid; e < n * octs; e += 256) {
        const int t = first + e / octs, d0 = 8 * (e % octs);
        const float* row = q + (size_t)t * ldq + (size_t)h * dk;
        uint4 u;
        if (d0 < dim) {
            const float* p = row + d0;
            u = make_uint4(pack_bf16(p[0], p[1]), pack_bf16(p[2], p[3]), pack_bf16(p[4], p[5]), pack_bf16(p[6], p[7]));
        } else {
            u = rotated_oct(row + dim, d0 - dim, rot, rot_dims, pairing, cs + (size_t)t * half);
        }
        *reinterpret_cast<uint4*>(q_out + ((size_t)t * H + h) * dk + d0) = u;
    }
}

LLOGOS_EXPORT int llogos_latent_heads(const void* kvh, const float* kv, int ldkv, int rank, const float* q, int ldq, const void* cs,
                                      void* q_out, void* k_pool, void* v_pool, const int* table, int table_stride, const int* cu,
                                      int batch, int n_pages, int H, int dim, int rot, int rot_dims, int pairing, int dv,
                                      hipStream_t stream) {
    if (batch <= 0 || n_pages <= 0 || H <= 0 || dim <= 0 || rot < 0 || dv <= 0 || dim % 8 || rot % 8 || (dim + rot) % 16 || dv % 16) return LLOGOS_BAD_ARGUMENT;
    if (rot_dims < 0 || rot_dims > rot || rot_dims % 2 || (pairing != 0 && pairing != 1) || (rot_dims && !cs)) return LLOGOS_BAD_ARGUMENT;
    if (ldkv < rank + rot || ldq < H * (dim + rot) || (uintptr_t)kvh % 16 || (uintptr_t)q_out % 16 || (uintptr_t)k_pool % 16 || (uintptr_t)v_pool % 16) return LLOGOS_BAD_ARGUMENT;
    latent_heads_kernel<<<dim3(n_pages, H), 256, 0, stream>>>((const bf16_t*)kvh, kv, ldkv, rank, q, ldq, (const float2*)cs, (bf16_t*)q_out,
        (bf16_t*)k_pool, (bf16_t*)v_pool, table, table_stride, cu, batch, H, dim, rot, rot_dims, pairing, dv);
    return LLOGOS_LAUNCH_CHECK();
}

// The 128-row prompt kernel for keys of 64, 96, 128 or 192 and values of 64, 80, 96 or 128 dimensions.  Plain softmax with
// or without a window; with head_sink or gate (no window then) the form that finishes its rows with them, built for keys
// of 192 (the others are in capped_attention_mfma_bf16.hip).  -2: a shape or a combination that is not built.
LLOGOS_EXPORT int llogos_wide_attn_prefill_bf16(void* out, const void* q, int q_stride, const void* k_pool, const void* v_pool,
                                                const int* table, int table_stride, const int* cu, const int* tok_pos, int batch,
                                                int n_tiles, int n_heads, int n_kv_heads, int dk, int dv, float scale, int window,
                                                const float* head_sink, const float* gate, int gate_stride, int halves,
                                                hipStream_t stream) {
    if (batch <= 0 || n_tiles <= 0 || window < 0 || n_heads <= 0 || n_kv_heads <= 0 || n_heads % n_kv_heads || (gate && gate_stride < n_heads)) return LLOGOS_BAD_ARGUMENT;
    if (halves != 1 && halves != 2) return LLOGOS_BAD_ARGUMENT;
    const bool bent = head_sink || gate;
    if (q_stride % 8 || n_heads / n_kv_heads > 16 || (bent && (window > 0 || dk != 192))) return LLOGOS_UNSUPPORTED;
    if (dk == 192) halves = 1;                   // (two sets of page buffers would take all of a unit's LDS)
    const int group = n_heads / n_kv_heads;
    const long long pairs = (long long)n_tiles * n_kv_heads;
    const dim3 grid((unsigned)((pairs + 7) / 8 * 8 * group));
#define WIDE(KS, VB, HALVES, BENT) do { \
        size_t smem = HALVES * 2 * sizeof(DirectPageLds<32 * KS, 16 * VB>); \
        if (HALVES == 2) smem = std::max(smem, (size_t)kAttnWaves * 2 * (2 + 4 * VB) * kWave * sizeof(float)); \
        hipError_t e = hipFuncSetAttribute((const void*)attn_prefill_direct_kernel<32 * KS, HALVES, 16 * VB, BENT>, \
                                           hipFuncAttributeMaxDynamicSharedMemorySize, (int)smem); \
        if (e != hipSuccess) return (int)e; \
        attn_prefill_direct_kernel<32 * KS, HALVES, 16 * VB, BENT><<<grid, HALVES * kAttnWaves * kWave, smem, stream>>>( \
            (bf16_t*)out, (const bf16_t*)q, q_stride, (const bf16_t*)k_pool, (const bf16_t*)v_pool, table, table_stride, \
            cu, tok_pos, batch, n_tiles, n_heads, n_kv_heads, group, scale, window, 0, 0.f, head_sink, gate, gate_stride); \
        return LLOGOS_LAUNCH_CHECK(); } while (0)
#define WIDEV(KS, HALVES, BENT) do { if (dv == 64) WIDE(KS, 4, HALVES, BENT); else if (dv == 80) WIDE(KS, 5, HALVES, BENT); \
        else if (dv == 96) WIDE(KS, 6, HALVES, BENT); else if (dv == 128) WIDE(KS, 8, HALVES, BENT); else return LLOGOS_UNSUPPORTED; } while (0)
#define WIDEH(KS) do { if (halves == 2) WIDEV(KS, 2, false); else WIDEV(KS, 1, false); } while (0)
    if (dk == 192) { if (bent) WIDEV(6, 1, true); else WIDEV(6, 1, false); }
    if (dk == 64) WIDEH(2);
    if (dk == 96) WIDEH(3);
    if (dk == 128) WIDEH(4);
#undef WIDEH
#undef WIDEV
#undef WIDE
    return LLOGOS_UNSUPPORTED;
}
