// A linear recurrence with a matrix state per head whose decay is one fixed number a head, and the norm and
// gate behind it.  Per sequence and head, with S [key channel d, value channel c] carried from token to token:
//     q_t, k_t, v_t = silu of the projected rows
//     S <- a S + k_t v_t^T;   o_t[c] = sum_d q_t[d] S[d, c]
// Rows [q | k | v | ...] are float32 [T, ld] (q, k: heads x D; v: heads x V), maybe as `parts` partial sums of a
// product split along k; o is float32 [T, heads * V]; the state is float32, [heads][D][V] a slot.
// All sums and products are 32-bit.
//
// Two kernels: single-token steps stream the state once (a read and a write); longer steps go in chunks of 32
// tokens on the matrix cores' 32-bit products (v_mfma_f32_16x16x4_f32), in which, with i, j tokens of the chunk
// and n its length,
//     O^T = V^T A^T + S^T Q'^T,   A[i][j] = a^(i-j) q_i . k_j (j <= i),   Q'_i = a^(i+1) q_i
//     S  <- a^n S + sum_j a^(n-1-j) k_j v_j^T
// so that nothing but the chunk's end state is carried.  Powers of a come from a table made in double.
#include "common.h"

typedef float df32x4 __attribute__((ext_vector_type(4)));

constexpr int kDecayChunk = 32;            // tokens a chunk (the table of powers holds a^0 .. a^32)

__device__ __forceinline__ float decay_silu(float z) { return z / (1.0f + expf(-z)); }

// ---------------------------------------------------------------- single-token steps
// grid (sequences, heads, column blocks); a block owns `cols` columns of S (VEC neighbouring ones a thread), its
// threads are cols / VEC wide and P deep: thread p of a column walks rows p, p + P, ...; the P sums of a
// column meet in LDS.
template <int VEC>
__global__ __launch_bounds__(256) void decay_step_kernel(float* __restrict__ o, const float* __restrict__ rows, int ld, int parts,
                                                         size_t part_stride, const float* __restrict__ powers, float* __restrict__ state,
                                                         size_t state_stride, const int* __restrict__ slots, int H, int D, int V, int cols) {
    extern __shared__ float lds[];
    float* sq = lds;                       // [D]
    float* sk = sq + D;                    // [D]
    float* sum = sk + D;                   // [P][cols]
    const int seq = blockIdx.x, head = blockIdx.y, c0 = blockIdx.z * cols;
    const int tid = threadIdx.x;
    const float* row = rows + (size_t)seq * ld;
    const int width = cols / VEC, P = blockDim.x / width;
    const int p = tid / width, c = c0 + (tid % width) * VEC;
    const bool on = p < P && c < V;        // (V is a multiple of VEC)
    for (int d = tid; d < D; d += blockDim.x) {
        float zq = row[(size_t)head * D + d], zk = row[(size_t)(H + head) * D + d];
        for (int s = 1; s < parts; ++s) {
            zq += row[s * part_stride + (size_t)head * D + d];
            zk += row[s * part_stride + (size_t)(H + head) * D + d];
        }
        sq[d] = decay_silu(zq);
        sk[d] = decay_silu(zk);
    }
    float v[VEC], acc[VEC];
#pragma unroll
    for (int e = 0; e < VEC; ++e) {
        v[e] = acc[e] = 0.f;
        if (on) {
            const size_t at = (size_t)2 * H * D + (size_t)head * V + c + e;
            float z = row[at];
            for (int s = 1; s < parts; ++s) z += row[s * part_stride + at];
            v[e] = decay_silu(z);
        }
    }
    __syncthreads();
    const float a = powers[(size_t)head * (kDecayChunk + 1) + 1];
    float* S = state + (size_t)slots[seq] * state_stride + (size_t)head * D * V + c;
    if (on) {
        constexpr int AHEAD = 8;           // rows of the state on their way at a time
        for (int d0 = p; d0 < D; d0 += AHEAD * P) {
            float s[AHEAD][VEC];
#pragma unroll
            for (int r = 0; r < AHEAD; ++r) {
                const int d = d0 + r * P;
                if (d < D) {
                    if (VEC == 4) {
                        const float4 t = *reinterpret_cast<const float4*>(S + (size_t)d * V);
                        s[r][0] = t.x; s[r][1 % VEC] = t.y; s[r][2 % VEC] = t.z; s[r][3 % VEC] = t.w;
                    } else {
                        s[r][0] = S[(size_t)d * V];
                    }
                }
            }
#pragma unroll
            for (int r = 0; r < AHEAD; ++r) {
                const int d = d0 + r * P;
                if (d < D) {
                    const float k = sk[d], q = sq[d];
#pragma unroll
                    for (int e = 0; e < VEC; ++e) {
                        s[r][e] = fmaf(a, s[r][e], k * v[e]);
                        acc[e] = fmaf(q, s[r][e], acc[e]);
                    }
                    if (VEC == 4) *reinterpret_cast<float4*>(S + (size_t)d * V) = make_float4(s[r][0], s[r][1 % VEC], s[r][2 % VEC], s[r][3 % VEC]);
                    else S[(size_t)d * V] = s[r][0];
                }
            }
        }
    }
    if (p < P) {
#pragma unroll
        for (int e = 0; e < VEC; ++e) sum[(size_t)p * cols + (tid % width) * VEC + e] = acc[e];
    }
    __syncthreads();
    for (int i = tid; i < cols; i += blockDim.x) {
        if (c0 + i >= V) continue;
        float t = 0.f;
        for (int s = 0; s < P; ++s) t += sum[(size_t)s * cols + i];
        o[((size_t)seq * H + head) * V + c0 + i] = t;
    }
}

// ---------------------------------------------------------------- longer steps, chunk by chunk
// grid (sequences, heads, column blocks * segments), four waves; a wave owns VT tiles of 16 columns of S in the
// layout of a product's result (tile (dt, vt): lane (c = lane & 15, g = lane >> 4) holds rows 16 dt + 4 g .. + 3 of
// column c), which is also the layout of an operand whose k runs over those rows in the order 16 dt + 4 g + e, so the
// state never leaves the registers.  Every operand read from LDS is four neighbouring values of its k (16 bytes), and
// both operands of a product take k in that order.
// LDS rows are padded by four floats: sixteen rows times four 16-byte pieces then fall on different banks.
// MODE 0: a sequence from the cached state to the cached state.  Long prompts of few sequences are cut into segments
// that run side by side: MODE 1 takes a segment from a zero state and leaves its end state (no outputs);
// decay_combine_kernel turns those into every segment's initial state and the sequence's final one; MODE 2 runs
// the segment from its initial state for the outputs.
constexpr int kDecayPad = 4;

// tiles of D: DT = ceil(D / 16); LDS floats: Q and K [32][16 DT + 4], K^T [16 DT][36], V^T [64 VT][36], A [32][36]
__host__ __device__ constexpr int decay_lds_floats(int DT, int VT) {
    return 2 * kDecayChunk * (16 * DT + kDecayPad) + 16 * DT * (kDecayChunk + kDecayPad) + 64 * VT * (kDecayChunk + kDecayPad) +
           kDecayChunk * (kDecayChunk + kDecayPad);
}

template <int DT, int VT, int MODE>
__global__ __launch_bounds__(256) void decay_chunk_kernel(float* __restrict__ o, const float* __restrict__ rows, int ld, int parts,
                                                          size_t part_stride, const float* __restrict__ powers,
                                                          float* __restrict__ state, size_t state_stride, const int* __restrict__ slots,
                                                          const int* __restrict__ cu, int H, int D, int V, int col_blocks, int n_seg,
                                                          int seg_len, float* __restrict__ seg_state, int vec) {
    constexpr int C = kDecayChunk, DP = 16 * DT + kDecayPad, CP = C + kDecayPad, VB = 64 * VT;
    extern __shared__ __attribute__((aligned(16))) float lds[];
    float* sQ = lds;                       // [C][DP]   rows times a^(i + 1) where the state is read: the factor comes with the store of o
    float* sK = sQ + C * DP;               // [C][DP]
    float* sKT = sK + C * DP;              // [16 DT][CP], times a^(n - 1 - j)
    float* sVT = sKT + 16 * DT * CP;       // [VB][CP]
    float* sA = sVT + VB * CP;             // [C][CP]: A[i][j]
    __shared__ float pw[C + 1];
    const int seq = blockIdx.x, head = blockIdx.y, cb = blockIdx.z % col_blocks, seg = blockIdx.z / col_blocks;
    const int first0 = cu[seq], count0 = cu[seq + 1] - first0;
    const int first = first0 + (MODE ? seg * seg_len : 0);
    const int count = MODE ? min(seg_len, count0 - seg * seg_len) : count0;
    const int tid = threadIdx.x, lane = tid & (kWave - 1), wave = tid / kWave;
    const int c = lane & 15, g = lane >> 4;
    const int col0 = cb * VB + wave * 16 * VT;             // the wave's first column
    for (int i = tid; i <= C; i += 256) pw[i] = powers[(size_t)head * (C + 1) + i];

    float* S = MODE ? seg_state + (((size_t)seq * n_seg + seg) * H + head) * D * V
                    : state + (size_t)slots[seq] * state_stride + (size_t)head * D * V;
    df32x4 s[DT][VT];
#pragma unroll
    for (int dt = 0; dt < DT; ++dt)
#pragma unroll
        for (int vt = 0; vt < VT; ++vt)
#pragma unroll
            for (int r = 0; r < 4; ++r) {
                const int d = 16 * dt + 4 * g + r, col = col0 + 16 * vt + c;
                s[dt][vt][r] = (MODE != 1 && d < D && col < V) ? S[(size_t)d * V + col] : 0.f;
            }
    // four neighbouring values of a token's row, from column `at` on (those at or behind `end` are zeros), activated
    auto value4 = [&](int j, int n, size_t at, size_t end) {
        float4 z = make_float4(0.f, 0.f, 0.f, 0.f);
        if (j < n && at < end) {
            const float* p = rows + (size_t)(first + j) * ld + at;
            for (int q = 0; q < parts; ++q, p += part_stride) {
                if (vec) {
                    const float4 u = *reinterpret_cast<const float4*>(p);
                    z.x += u.x; z.y += u.y; z.z += u.z; z.w += u.w;
                } else {
                    z.x += p[0];
                    if (at + 1 < end) z.y += p[1];
                    if (at + 2 < end) z.z += p[2];
                    if (at + 3 < end) z.w += p[3];
                }
            }
            z = make_float4(decay_silu(z.x), decay_silu(z.y), decay_silu(z.z), decay_silu(z.w));
        }
        return z;
    };
    for (int t0 = 0; t0 < count; t0 += C) {
        const int n = min(C, count - t0);
        __syncthreads();                                   // the chunk before has been read (and pw is there)
        // (a wave takes 16 rows, 64 bytes of each: the transposed copies' stores then fall on neighbouring words of a row)
#pragma unroll 4
        for (int e = tid; e < C * 4 * DT; e += 256) {
            const int j = (e & 15) + 16 * ((e >> 4) / (4 * DT)), d = 4 * ((e >> 4) % (4 * DT));
            const float4 k = value4(t0 + j, t0 + n, (size_t)(H + head) * D + d, (size_t)(H + head + 1) * D);
            if (MODE != 1) {
                *reinterpret_cast<float4*>(sQ + j * DP + d) = value4(t0 + j, t0 + n, (size_t)head * D + d, (size_t)(head + 1) * D);
                *reinterpret_cast<float4*>(sK + j * DP + d) = k;
            }
            const float f = j < n ? pw[n - 1 - j] : 0.f;
            sKT[(d + 0) * CP + j] = k.x * f;
            sKT[(d + 1) * CP + j] = k.y * f;
            sKT[(d + 2) * CP + j] = k.z * f;
            sKT[(d + 3) * CP + j] = k.w * f;
        }
#pragma unroll 4
        for (int e = tid; e < C * VB / 4; e += 256) {
            const int j = (e & 15) + 16 * ((e >> 4) / (VB / 4)), i = 4 * ((e >> 4) % (VB / 4));
            const size_t v0 = (size_t)2 * H * D + (size_t)head * V;
            const float4 v = value4(t0 + j, t0 + n, v0 + cb * VB + i, v0 + V);
            sVT[(i + 0) * CP + j] = v.x;
            sVT[(i + 1) * CP + j] = v.y;
            sVT[(i + 2) * CP + j] = v.z;
            sVT[(i + 3) * CP + j] = v.w;
        }
        __syncthreads();
        if (MODE != 1) {
            // A^T, tile (jt, it): rows j, columns i; wave 0: (0, 0), wave 1: (0, 1), wave 2: (1, 1); above the diagonal nothing is
            if (wave < 3) {
                const int jt = wave == 2 ? 1 : 0, it = wave == 0 ? 0 : 1;
                df32x4 t = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
                for (int dt = 0; dt < DT; ++dt) {
                    const float4 ka = *reinterpret_cast<const float4*>(sK + (16 * jt + c) * DP + 16 * dt + 4 * g);
                    const float4 qb = *reinterpret_cast<const float4*>(sQ + (16 * it + c) * DP + 16 * dt + 4 * g);
                    t = __builtin_amdgcn_mfma_f32_16x16x4f32(ka.x, qb.x, t, 0, 0, 0);
                    t = __builtin_amdgcn_mfma_f32_16x16x4f32(ka.y, qb.y, t, 0, 0, 0);
                    t = __builtin_amdgcn_mfma_f32_16x16x4f32(ka.z, qb.z, t, 0, 0, 0);
                    t = __builtin_amdgcn_mfma_f32_16x16x4f32(ka.w, qb.w, t, 0, 0, 0);
                }
                const int i = 16 * it + c, j = 16 * jt + 4 * g;
                float4 w;
                w.x = j + 0 <= i ? t[0] * pw[i - j] : 0.f;
                w.y = j + 1 <= i ? t[1] * pw[i - j - 1] : 0.f;
                w.z = j + 2 <= i ? t[2] * pw[i - j - 2] : 0.f;
                w.w = j + 3 <= i ? t[3] * pw[i - j - 3] : 0.f;
                *reinterpret_cast<float4*>(sA + i * CP + j) = w;
            }
            __syncthreads();
            // O^T, tiles (vt, it): the state's share first, scaled by a^(i + 1), then the chunk's own
            df32x4 ot[VT][2];
#pragma unroll
            for (int vt = 0; vt < VT; ++vt) ot[vt][0] = ot[vt][1] = df32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
            for (int dt = 0; dt < DT; ++dt) {
#pragma unroll
                for (int it = 0; it < 2; ++it) {
                    const float4 qb = *reinterpret_cast<const float4*>(sQ + (16 * it + c) * DP + 16 * dt + 4 * g);
#pragma unroll
                    for (int vt = 0; vt < VT; ++vt) {
                        ot[vt][it] = __builtin_amdgcn_mfma_f32_16x16x4f32(s[dt][vt][0], qb.x, ot[vt][it], 0, 0, 0);
                        ot[vt][it] = __builtin_amdgcn_mfma_f32_16x16x4f32(s[dt][vt][1], qb.y, ot[vt][it], 0, 0, 0);
                        ot[vt][it] = __builtin_amdgcn_mfma_f32_16x16x4f32(s[dt][vt][2], qb.z, ot[vt][it], 0, 0, 0);
                        ot[vt][it] = __builtin_amdgcn_mfma_f32_16x16x4f32(s[dt][vt][3], qb.w, ot[vt][it], 0, 0, 0);
                    }
                }
            }
#pragma unroll
            for (int it = 0; it < 2; ++it) {
                const float f = pw[16 * it + c + 1];
#pragma unroll
                for (int vt = 0; vt < VT; ++vt)
#pragma unroll
                    for (int r = 0; r < 4; ++r) ot[vt][it][r] *= f;
            }
#pragma unroll
            for (int it = 0; it < 2; ++it)
#pragma unroll
                for (int jt = 0; jt <= it; ++jt) {
                    const float4 ab = *reinterpret_cast<const float4*>(sA + (16 * it + c) * CP + 16 * jt + 4 * g);
#pragma unroll
                    for (int vt = 0; vt < VT; ++vt) {
                        const float4 va = *reinterpret_cast<const float4*>(sVT + (wave * 16 * VT + 16 * vt + c) * CP + 16 * jt + 4 * g);
                        ot[vt][it] = __builtin_amdgcn_mfma_f32_16x16x4f32(va.x, ab.x, ot[vt][it], 0, 0, 0);
                        ot[vt][it] = __builtin_amdgcn_mfma_f32_16x16x4f32(va.y, ab.y, ot[vt][it], 0, 0, 0);
                        ot[vt][it] = __builtin_amdgcn_mfma_f32_16x16x4f32(va.z, ab.z, ot[vt][it], 0, 0, 0);
                        ot[vt][it] = __builtin_amdgcn_mfma_f32_16x16x4f32(va.w, ab.w, ot[vt][it], 0, 0, 0);
                    }
                }
#pragma unroll
            for (int it = 0; it < 2; ++it) {
                const int i = 16 * it + c;
                if (i >= n) continue;
                float* orow = o + ((size_t)(first + t0 + i) * H + head) * V;
#pragma unroll
                for (int vt = 0; vt < VT; ++vt) {
                    const int col = col0 + 16 * vt + 4 * g;
                    if ((V & 3) == 0) {
                        if (col < V) *reinterpret_cast<float4*>(orow + col) = make_float4(ot[vt][it][0], ot[vt][it][1], ot[vt][it][2], ot[vt][it][3]);
                    } else {
#pragma unroll
                        for (int r = 0; r < 4; ++r)
                            if (col + r < V) orow[col + r] = ot[vt][it][r];
                    }
                }
            }
        }
        // the state behind the chunk
        const float an = pw[n];
        float4 vb[VT][2];
#pragma unroll
        for (int vt = 0; vt < VT; ++vt)
#pragma unroll
            for (int jt = 0; jt < 2; ++jt) vb[vt][jt] = *reinterpret_cast<const float4*>(sVT + (wave * 16 * VT + 16 * vt + c) * CP + 16 * jt + 4 * g);
#pragma unroll
        for (int dt = 0; dt < DT; ++dt) {
#pragma unroll
            for (int vt = 0; vt < VT; ++vt)
#pragma unroll
                for (int r = 0; r < 4; ++r) s[dt][vt][r] *= an;
#pragma unroll
            for (int jt = 0; jt < 2; ++jt) {
                const float4 ka = *reinterpret_cast<const float4*>(sKT + (16 * dt + c) * CP + 16 * jt + 4 * g);
#pragma unroll
                for (int vt = 0; vt < VT; ++vt) {
                    s[dt][vt] = __builtin_amdgcn_mfma_f32_16x16x4f32(ka.x, vb[vt][jt].x, s[dt][vt], 0, 0, 0);
                    s[dt][vt] = __builtin_amdgcn_mfma_f32_16x16x4f32(ka.y, vb[vt][jt].y, s[dt][vt], 0, 0, 0);
                    s[dt][vt] = __builtin_amdgcn_mfma_f32_16x16x4f32(ka.z, vb[vt][jt].z, s[dt][vt], 0, 0, 0);
                    s[dt][vt] = __builtin_amdgcn_mfma_f32_16x16x4f32(ka.w, vb[vt][jt].w, s[dt][vt], 0, 0, 0);
                }
            }
        }
    }
    if (MODE == 2) return;
#pragma unroll
    for (int dt = 0; dt < DT; ++dt)
#pragma unroll
        for (int vt = 0; vt < VT; ++vt)
#pragma unroll
            for (int r = 0; r < 4; ++r) {
                const int d = 16 * dt + 4 * g + r, col = col0 + 16 * vt + c;
                if (d < D && col < V) S[(size_t)d * V + col] = s[dt][vt][r];
            }
}

// The segments' local end states chained: seg_state[seg] <- the state the segment starts from, and the cached state
// <- the state after the last segment; a segment of n tokens decays what was before it by a^n (n by repeated
// factors a^32 and the rest from the table).  A thread owns an element of S.
__global__ void decay_combine_kernel(float* __restrict__ state, size_t state_stride, const int* __restrict__ slots,
                                     float* __restrict__ seg_state, const float* __restrict__ powers, const int* __restrict__ cu,
                                     int H, int size, int n_seg, int seg_len) {
    const int seq = blockIdx.x, head = blockIdx.y;
    const float* pw = powers + (size_t)head * (kDecayChunk + 1);
    const int e = blockIdx.z * blockDim.x + threadIdx.x;
    if (e >= size) return;
    const int count = cu[seq + 1] - cu[seq];
    float whole = 1.f;
    for (int i = 0; i < seg_len; i += kDecayChunk) whole *= pw[kDecayChunk];          // (seg_len is whole chunks)
    float* S = state + (size_t)slots[seq] * state_stride + (size_t)head * size + e;
    float cur = *S;
    for (int sg = 0; sg < n_seg; ++sg) {
        const int n = min(seg_len, count - sg * seg_len);
        if (n <= 0) break;
        float* at = seg_state + (((size_t)seq * n_seg + sg) * H + head) * size + e;
        const float local = *at;
        *at = cur;
        float f = whole;
        if (n < seg_len) {
            f = pw[n % kDecayChunk];
            for (int i = 0; i < n / kDecayChunk; ++i) f *= pw[kDecayChunk];
        }
        cur = fmaf(f, cur, local);
    }
    *S = cur;
}

// cu null: a single-token step.  powers float [H][33]: a^0 .. a^32 of every head.  seg_state (n_seg > 1): float
// [sequences][n_seg][H][D][V]; seg_len a multiple of 32.
LLOGOS_EXPORT int llogos_decay_scan(float* o, const float* rows, int ld, int parts, long long part_stride, const float* powers,
                                    float* state, long long state_stride, const int* slots, const int* cu, int B, int H, int D, int V,
                                    int step_cols, int n_seg, int seg_len, float* seg_state, hipStream_t stream) {
    if (B <= 0 || H <= 0 || D <= 0 || V <= 0 || parts < 1 || ld < 2 * H * D + H * V || n_seg < 1) return LLOGOS_BAD_ARGUMENT;
    if (state_stride < (long long)H * D * V || D > 256) return LLOGOS_BAD_ARGUMENT;
    if (!cu) {
        const bool vec = V % 4 == 0 && state_stride % 4 == 0 && (uintptr_t)state % 16 == 0;
        if (step_cols < 4 || step_cols % 4 || step_cols > 256) return LLOGOS_BAD_ARGUMENT;
        const int width = vec ? step_cols / 4 : step_cols, P = 256 / width;
        dim3 grid(B, H, (V + step_cols - 1) / step_cols);
        const size_t smem = (size_t)(2 * D + P * step_cols) * sizeof(float);
        if (vec) decay_step_kernel<4><<<grid, width * P, smem, stream>>>(o, rows, ld, parts, (size_t)part_stride, powers, state, (size_t)state_stride, slots, H, D, V, step_cols);
        else decay_step_kernel<1><<<grid, width * P, smem, stream>>>(o, rows, ld, parts, (size_t)part_stride, powers, state, (size_t)state_stride, slots, H, D, V, step_cols);
        return LLOGOS_LAUNCH_CHECK();
    }
    if (n_seg > 1 && (!seg_state || seg_len < kDecayChunk || seg_len % kDecayChunk)) return LLOGOS_BAD_ARGUMENT;
    if (n_seg == 1) seg_len = 0;
    const int dt = (D + 15) / 16, vt = V > 64 ? 2 : 1;
    const int col_blocks = (V + 64 * vt - 1) / (64 * vt);
    dim3 grid(B, H, col_blocks * n_seg);
    const int vec4 = D % 4 == 0 && V % 4 == 0 && ld % 4 == 0 && part_stride % 4 == 0 && (uintptr_t)rows % 16 == 0 ? 1 : 0;
#define DC(DT, VT, MODE) do { \
        const int smem = decay_lds_floats(DT, VT) * (int)sizeof(float); \
        if (smem > 48 * 1024) { \
            hipError_t e = hipFuncSetAttribute((const void*)decay_chunk_kernel<DT, VT, MODE>, hipFuncAttributeMaxDynamicSharedMemorySize, smem); \
            if (e != hipSuccess) return (int)e; \
        } \
        decay_chunk_kernel<DT, VT, MODE><<<grid, 256, smem, stream>>>(o, rows, ld, parts, (size_t)part_stride, powers, state, \
            (size_t)state_stride, slots, cu, H, D, V, col_blocks, n_seg, seg_len, seg_state, vec4); } while (0)
#define DCM(DT, VT) do { \
        if (n_seg == 1) { DC(DT, VT, 0); break; } \
        DC(DT, VT, 1); \
        decay_combine_kernel<<<dim3(B, H, (D * V + 255) / 256), 256, 0, stream>>>(state, (size_t)state_stride, slots, seg_state, powers, cu, H, D * V, n_seg, seg_len); \
        DC(DT, VT, 2); } while (0)
#define DCV(DT) do { if (vt == 1) DCM(DT, 1); else DCM(DT, 2); } while (0)
    if (dt <= 1) DCV(1); else if (dt <= 2) DCV(2); else if (dt <= 4) DCV(4); else if (dt <= 6) DCV(6); else if (dt <= 8) DCV(8); else DCV(16);
#undef DCV
#undef DCM
#undef DC
    return LLOGOS_LAUNCH_CHECK();
}

// ---------------------------------------------------------------- norm over a row, weight, gate
// y[t, :] = o[t, :] / sqrt(mean(o[t, :]^2) + eps) * w * sigmoid(gate[t, :]); one block a row.  gate: float logits of row
// stride ldg, maybe in parts.  VEC: four neighbouring values a thread.
template <typename TO, int VEC>
__global__ __launch_bounds__(1024) void gated_row_norm_kernel(TO* __restrict__ y, const float* __restrict__ o, const float* __restrict__ w,
                                                              const float* __restrict__ gate, int ldg, int parts, size_t part_stride,
                                                              float eps, int N) {
    __shared__ float red[16];
    const int t = blockIdx.x;
    const float* row = o + (size_t)t * N;
    float ss = 0.f;
    for (int i = VEC * threadIdx.x; i < N; i += VEC * blockDim.x) {
        if (VEC == 4) {
            const float4 v = *reinterpret_cast<const float4*>(row + i);
            ss = fmaf(v.x, v.x, ss); ss = fmaf(v.y, v.y, ss); ss = fmaf(v.z, v.z, ss); ss = fmaf(v.w, v.w, ss);
        } else {
            ss = fmaf(row[i], row[i], ss);
        }
    }
    const float inv = 1.0f / sqrtf(block_sum(ss, red) / (float)N + eps);
    for (int i = VEC * threadIdx.x; i < N; i += VEC * blockDim.x) {
        float v[VEC], z[VEC], f[VEC];
        auto load = [&](float (&to)[VEC], const float* p) {
            if (VEC == 4) {
                const float4 u = *reinterpret_cast<const float4*>(p);
                to[0] = u.x; to[1 % VEC] = u.y; to[2 % VEC] = u.z; to[3 % VEC] = u.w;
            } else {
                to[0] = *p;
            }
        };
        load(v, row + i);
        load(f, w + i);
        load(z, gate + (size_t)t * ldg + i);
        for (int q = 1; q < parts; ++q) {
            float more[VEC];
            load(more, gate + q * part_stride + (size_t)t * ldg + i);
#pragma unroll
            for (int e = 0; e < VEC; ++e) z[e] += more[e];
        }
#pragma unroll
        for (int e = 0; e < VEC; ++e) store_f32(y + (size_t)t * N + i + e, v[e] * inv * f[e] * (1.0f / (1.0f + expf(-z[e]))));
    }
}

LLOGOS_EXPORT int llogos_gated_row_norm(void* y, int y_dtype, const float* o, const float* w, const float* gate, int ldg, int parts,
                                        long long part_stride, float eps, int T, int N, hipStream_t stream) {
    if (T <= 0 || N <= 0 || parts < 1 || ldg < N) return LLOGOS_BAD_ARGUMENT;
    const bool vec = N % 4 == 0 && ldg % 4 == 0 && part_stride % 4 == 0 && (uintptr_t)gate % 16 == 0 && (uintptr_t)o % 16 == 0 && (uintptr_t)w % 16 == 0;
    const int work = vec ? (N + 3) / 4 : N;
    const int threads = min(T >= 256 ? 256 : 1024, (work + kWave - 1) / kWave * kWave);
#define GRN(TO, V_) gated_row_norm_kernel<TO, V_><<<T, threads, 0, stream>>>((TO*)y, o, w, gate, ldg, parts, (size_t)part_stride, eps, N)
    if (y_dtype == DT_F32) { if (vec) GRN(float, 4); else GRN(float, 1); }
    else if (y_dtype == DT_BF16) { if (vec) GRN(bf16_t, 4); else GRN(bf16_t, 1); }
    else return LLOGOS_BAD_ARGUMENT;
#undef GRN
    return LLOGOS_LAUNCH_CHECK();
}
