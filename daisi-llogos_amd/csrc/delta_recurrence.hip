// A recurrence with a matrix state per head that is corrected rather than added to (the gated delta rule), with
// everything in front of it and behind it.  Per sequence and head, S [key channel d, value channel c]:
//     q, k, v   a short causal convolution over time of the projected rows, channel by channel, then silu;
//               q and k divided by sqrt(sum of squares + 1e-6) over a head's D channels, q also by sqrt(D)
//     g         exp(-exp(A_log) * softplus(z + dt_bias)), one number a head or one a key channel
//     S <- diag(g) S;   u = sigmoid(b) * (v - S^T k);   S <- S + k u^T;   o = S^T q
//     y         o / sqrt(mean(o^2) + eps) * w * silu(gate)  or  * sigmoid(gate)   over a head's V channels
// Head h reads the key head h / (H / G).  Rows are float32 [q (G D) | k (G D) | v (H V) | ...], row stride ld, maybe
// as `parts` partial sums of a product split along k.  All arithmetic is 32-bit.
//
// A slot's state row holds S of every head, [H][D][V], and behind it the convolution's ring: [taps][W] with W = 2 G D + H V,
// whose row p % taps holds the projected row of position p.  A step writes rows that none of its readers reads (the
// row of position p - taps is gone when p comes), so blocks that share a key head need no order among them.
//
// Single-token steps are one kernel (delta_step_kernel).  Longer steps go in chunks of 32 tokens: with b_i the sum of
// the logarithms of g from the chunk's first token to token i (a number a head or a key channel),
//     A_ij = beta_i sum_d k_id k_jd exp(b_i - b_j)   (j < i),      P_ij = sum_d q_id k_jd exp(b_i - b_j)   (j <= i)
//     T = (I + A)^-1,   M = P T,   K'_j = beta_j k_j exp(b_j),   V'_j = beta_j v_j
//     U = T V' - (T K') S,     O = M V' + (q exp(b) - M K') S,     S <- diag(exp(b_n)) S + (k exp(b_n - b))^T U
// T V', -T K', M V', q exp(b) - M K' and k exp(b_n - b) do not depend on S: delta_chunk_kernel makes them for all chunks
// side by side, and delta_scan_kernel walks a sequence's chunks with two products with S and one update each, on
// v_mfma_f32_16x16x4_f32 throughout.  No exponent is ever positive: a quotient of decays is taken as the exponential of
// the difference within 16 tokens, or as two factors that meet between two runs of 16 tokens.
#include "common.h"

typedef float dl4 __attribute__((ext_vector_type(4)));

constexpr int kDeltaChunk = 32;
constexpr int kDeltaMaxTaps = 16;
constexpr int kDeltaMaxDim = 256;         // key channels a head
constexpr int kDeltaMaxV = 1024;          // value channels a head
constexpr int kDeltaPad = 4;
constexpr int kDeltaCP = kDeltaChunk + kDeltaPad;
constexpr float kDeltaLog2e = 1.4426950408889634f;
constexpr float kDeltaFloor = -120.0f;    // a token's decay is at least 2^-120

__device__ __forceinline__ float delta_silu(float z) { return z / (1.0f + expf(-z)); }
__device__ __forceinline__ float delta_sigmoid(float z) { return 1.0f / (1.0f + expf(-z)); }
__device__ __forceinline__ float delta_exp2(float x) { return __builtin_amdgcn_exp2f(x); }

// log2 of a token's decay
__device__ __forceinline__ float delta_log_decay(float z, float a_log) {
    const float sp = fmaxf(z, 0.f) + log1pf(expf(-fabsf(z)));
    return fmaxf(-expf(a_log) * sp * kDeltaLog2e, kDeltaFloor);
}

__device__ __forceinline__ float delta_sum_parts(const float* p, int parts, size_t part_stride) {
    float v = p[0];
    for (int q0 = 1; q0 < parts; q0 += 4) {               // four loads in flight, added in ascending order
        float y[4];
#pragma unroll
        for (int j = 0; j < 4; ++j) y[j] = q0 + j < parts ? p[(size_t)(q0 + j) * part_stride] : 0.f;
#pragma unroll
        for (int j = 0; j < 4; ++j)
            if (q0 + j < parts) v += y[j];
    }
    return v;
}

// What the kernels are told about a step's projected rows and the sequences' state.
struct DeltaRows {
    const float* rows;          // [parts][T][ld]
    int ld, parts;
    size_t part_stride;
    const float* conv;          // [taps][W], the last row multiplies the token's own row
    int taps, W;
    float* state;
    size_t state_stride, ring;  // floats from a slot's row to the next, and from its start to the ring
    const int* slots;
    const int* tok_pos;
    int H, G, D, V;
};

// the decay's and beta's inputs: z (float, maybe in parts) at column z_col of rows of ldz, dt_bias, A_log [H]
struct DeltaGates {
    const float* z;
    int ldz, z_parts;
    size_t z_part_stride;
    const float* dt_bias;
    const float* a_log;
    int channelwise;            // z and dt_bias hold H D numbers, else H
    int b_col;                  // column of beta's logits in the projected rows
};

// channel c of the row `back` tokens before token t (of its sequence's `before`-th in the step), at position pos - back
__device__ __forceinline__ float delta_input(const DeltaRows& r, const float* ring, int t, int pos, int before, int back, int c) {
    if (back <= before) return delta_sum_parts(r.rows + (size_t)(t - back) * r.ld + c, r.parts, r.part_stride);
    return pos >= back ? ring[(size_t)((pos - back) % r.taps) * r.W + c] : 0.f;
}

// ---------------------------------------------------------------- single-token steps
// One block a (sequence, head).  Thread (p, x) holds VEC neighbouring columns of rows p, p + P, ... of S in registers from
// the first load to the store; both column sums S^T k and S^T q come from one pass, since with k . q known
// o = (g S)^T q + (k . q) u.
// A block's time is the latency of its loads, so all that a thread needs (its share of S, a channel of q, of k and of v with
// the rows before them, its decay, beta, the gate) is asked for before the first sum; up to four taps and four parts of
// a product that way (TAPS 4), more in loops.
template <int VEC, int RPT, int NT, int TAPS, typename TO>
__global__ __launch_bounds__(NT) void delta_step_kernel(TO* __restrict__ y, DeltaRows in, DeltaGates gt, const float* __restrict__ gate,
                                                        int ldg, int gate_parts, size_t gate_part_stride, int gate_silu,
                                                        const float* __restrict__ norm_w, float eps) {
    extern __shared__ float lds[];
    __shared__ float red[3][16];
    const int D = in.D, V = in.V, H = in.H, G = in.G;
    const int width = (V + VEC - 1) / VEC, P = blockDim.x / width;
    float* sq = lds;                       // [D]
    float* sk = sq + D;                    // [D]
    float* sg = sk + D;                    // [D]
    float* sv = sg + D;                    // [V]
    float* sz = sv + V;                    // [V] the gate's logits
    float* su = sz + V;                    // [width VEC]
    float* sum = su + width * VEC;         // [2][P][width VEC]
    const int seq = blockIdx.x, head = blockIdx.y, kvh = head / (H / G);
    const int tid = threadIdx.x, p = tid / width, c0 = (tid % width) * VEC;
    const bool on = p < P;
    const int pos = in.tok_pos[seq];
    float* slot = in.state + (size_t)in.slots[seq] * in.state_stride;
    float* ring = slot + in.ring;
    float* S = slot + (size_t)head * D * V + c0;
    const int turn = pos % in.taps;        // the ring's row of this position

    float s[RPT][VEC];
#pragma unroll
    for (int r = 0; r < RPT; ++r) {
        const int d = p + r * P;
        if (on && d < D) {
            if (VEC == 4) {
                const float4 t = *reinterpret_cast<const float4*>(S + (size_t)d * V);
                s[r][0] = t.x; s[r][1 % VEC] = t.y; s[r][2 % VEC] = t.z; s[r][3 % VEC] = t.w;
            } else {
                s[r][0] = S[(size_t)d * V];
            }
        } else {
#pragma unroll
            for (int e = 0; e < VEC; ++e) s[r][e] = 0.f;
        }
    }
    // the threads take channels of q and k from the front and of v from the back (D and V are at most blockDim)
    const int d = min(tid, D - 1), vi = (int)blockDim.x - 1 - tid, v_at = min(vi, V - 1);
    const bool has_k = tid < D, has_v = vi < V;
    const int chan[3] = {kvh * D + d, (G + kvh) * D + d, 2 * G * D + head * V + v_at};
    const float* row = in.rows + (size_t)seq * in.ld;
    const int zc = gt.channelwise ? head * D + d : head;
    const float* zp = gt.z + (size_t)seq * gt.ldz + zc;
    const float* gp = gate + (size_t)seq * ldg + head * V + v_at;
    const float* bp = row + gt.b_col + head;
    auto ask = [](const float* q, int parts, size_t stride, float (&to)[4]) {
#pragma unroll
        for (int j = 0; j < 4; ++j) to[j] = q[(size_t)min(j, parts - 1) * stride];
    };
    auto total = [](const float* q, int parts, size_t stride, const float (&from)[4]) {
        float v = from[0];
#pragma unroll
        for (int j = 1; j < 4; ++j) v += j < parts ? from[j] : 0.f;
        for (int j = 4; j < parts; ++j) v += q[(size_t)j * stride];
        return v;
    };
    float raw[3], act[3], z, z_out, b_logit;
    const float dt_bias = gt.dt_bias[zc], a_log = gt.a_log[head];
    if (TAPS == 4) {
        float x0[3][4], xs[3][4], w[3][4], zq[4], gq[4], bq[4];
#pragma unroll
        for (int i = 0; i < 3; ++i) {
            ask(row + chan[i], in.parts, in.part_stride, x0[i]);
#pragma unroll
            for (int j = 0; j < 4; ++j) {                  // the row `j` positions back and its tap
                const int back = min(j, in.taps - 1), at = turn - back + (turn < back ? in.taps : 0);
                w[i][j] = in.conv[(size_t)(in.taps - 1 - back) * in.W + chan[i]];
                xs[i][j] = j > 0 ? ring[(size_t)at * in.W + chan[i]] : 0.f;
            }
        }
        ask(zp, gt.z_parts, gt.z_part_stride, zq);
        ask(gp, gate_parts, gate_part_stride, gq);
        ask(bp, in.parts, in.part_stride, bq);
#pragma unroll
        for (int i = 0; i < 3; ++i) {
            raw[i] = total(row + chan[i], in.parts, in.part_stride, x0[i]);
            float acc = raw[i] * w[i][0];
#pragma unroll
            for (int j = 1; j < 4; ++j) acc = fmaf(w[i][j], (j < in.taps && pos >= j) ? xs[i][j] : 0.f, acc);
            act[i] = delta_silu(acc);
        }
        z = total(zp, gt.z_parts, gt.z_part_stride, zq);
        z_out = total(gp, gate_parts, gate_part_stride, gq);
        b_logit = total(bp, in.parts, in.part_stride, bq);
    } else {
#pragma unroll
        for (int i = 0; i < 3; ++i) {
            raw[i] = delta_sum_parts(row + chan[i], in.parts, in.part_stride);
            float acc = raw[i] * in.conv[(size_t)(in.taps - 1) * in.W + chan[i]];
            for (int j = 1; j < in.taps; ++j)
                if (pos >= j) acc = fmaf(in.conv[(size_t)(in.taps - 1 - j) * in.W + chan[i]],
                                         ring[(size_t)(turn - j + (turn < j ? in.taps : 0)) * in.W + chan[i]], acc);
            act[i] = delta_silu(acc);
        }
        z = delta_sum_parts(zp, gt.z_parts, gt.z_part_stride);
        z_out = delta_sum_parts(gp, gate_parts, gate_part_stride);
        b_logit = delta_sum_parts(bp, in.parts, in.part_stride);
    }
    const float beta = delta_sigmoid(b_logit);
    float qq = 0.f, kk = 0.f, qk = 0.f;
    if (has_k) {
        sq[d] = act[0];
        sk[d] = act[1];
        sg[d] = delta_exp2(delta_log_decay(z + dt_bias, a_log));
        qq = act[0] * act[0]; kk = act[1] * act[1]; qk = act[0] * act[1];
    }
    if (has_v) {
        sv[vi] = act[2];
        sz[vi] = z_out;
    }
    qq = wave_sum(qq); kk = wave_sum(kk); qk = wave_sum(qk);
    const int lane = tid & (kWave - 1), wave = tid / kWave, nwaves = blockDim.x / kWave;
    if (lane == 0) { red[0][wave] = qq; red[1][wave] = kk; red[2][wave] = qk; }
    __syncthreads();
    qq = kk = qk = 0.f;
    for (int w = 0; w < nwaves; ++w) { qq += red[0][w]; kk += red[1][w]; qk += red[2][w]; }
    const float qs = 1.0f / sqrtf(qq + 1e-6f) / sqrtf((float)D), ks = 1.0f / sqrtf(kk + 1e-6f);
    const float kq = qk * qs * ks;
    float ak[VEC], aq[VEC];
#pragma unroll
    for (int e = 0; e < VEC; ++e) ak[e] = aq[e] = 0.f;
#pragma unroll
    for (int r = 0; r < RPT; ++r) {
        const int d = p + r * P;
        if (on && d < D) {
            const float g = sg[d], k = sk[d], q = sq[d];
#pragma unroll
            for (int e = 0; e < VEC; ++e) {
                s[r][e] *= g;
                ak[e] = fmaf(k, s[r][e], ak[e]);
                aq[e] = fmaf(q, s[r][e], aq[e]);
            }
        }
    }
    if (on) {
#pragma unroll
        for (int e = 0; e < VEC; ++e) {
            sum[(size_t)p * width * VEC + c0 + e] = ak[e];
            sum[(size_t)(P + p) * width * VEC + c0 + e] = aq[e];
        }
    }
    __syncthreads();
    float o = 0.f;
    if (tid < V) {
        float rk = 0.f, rq = 0.f;
        for (int w = 0; w < P; ++w) {
            rk += sum[(size_t)w * width * VEC + tid];
            rq += sum[(size_t)(P + w) * width * VEC + tid];
        }
        const float u = beta * (sv[tid] - ks * rk);
        su[tid] = ks * u;
        o = fmaf(kq, u, qs * rq);
    }
    const float inv = 1.0f / sqrtf(block_sum(o * o, red[0]) / (float)V + eps);      // (its barriers also publish su)
    if (tid < V)
        store_f32(y + ((size_t)seq * H + head) * V + tid, o * inv * norm_w[tid] * (gate_silu ? delta_silu(sz[tid]) : delta_sigmoid(sz[tid])));
    // the token's projected channels join the ring (those of a key head once)
    if (has_k && head % (H / G) == 0) {
        ring[(size_t)turn * in.W + chan[0]] = raw[0];
        ring[(size_t)turn * in.W + chan[1]] = raw[1];
    }
    if (has_v) ring[(size_t)turn * in.W + chan[2]] = raw[2];
#pragma unroll
    for (int r = 0; r < RPT; ++r) {
        const int d = p + r * P;
        if (on && d < D) {
            const float k = sk[d];
#pragma unroll
            for (int e = 0; e < VEC; ++e) s[r][e] = fmaf(k, su[c0 + e], s[r][e]);
            if (VEC == 4) *reinterpret_cast<float4*>(S + (size_t)d * V) = make_float4(s[r][0], s[r][1 % VEC], s[r][2 % VEC], s[r][3 % VEC]);
            else S[(size_t)d * V] = s[r][0];
        }
    }
}

static bool delta_rows_ok(int ld, int parts, int taps, long long state_stride, int H, int G, int D, int V) {
    if (H <= 0 || G <= 0 || H % G || D <= 0 || V <= 0 || D > kDeltaMaxDim || V > kDeltaMaxV || parts < 1) return false;
    if (taps < 1 || taps > kDeltaMaxTaps) return false;
    const long long W = 2LL * G * D + (long long)H * V;
    return ld >= W && state_stride >= (long long)H * D * V + taps * W;
}

// threads a block: so few that a thread's share of S fits its registers (64 values), at least V
static int delta_step_threads(int D, int V, int vec) {
    const int width = (V + vec - 1) / vec;
    for (int t = 256; t <= 1024; t *= 2) {
        if (t < V) continue;
        const int P = t / width;
        if ((D + P - 1) / P * vec <= 64) return t;
    }
    return 0;
}

// Whether single-token steps are served at a head of D key and V value channels: threads a block, 0: no.
LLOGOS_EXPORT int llogos_delta_step_threads(int D, int V) {
    if (D <= 0 || V <= 0 || D > kDeltaMaxDim || V > kDeltaMaxV) return 0;
    return delta_step_threads(D, V, V % 4 == 0 ? 4 : 1);
}

LLOGOS_EXPORT int llogos_delta_step(void* y, int y_dtype, const float* rows, int ld, int parts, long long part_stride, const float* conv,
                                    int taps, float* state, long long state_stride, const int* slots, const int* tok_pos, int B, int H,
                                    int G, int D, int V, const float* z, int ldz, int z_parts, long long z_part_stride,
                                    const float* dt_bias, const float* a_log, int channelwise, int b_col, const float* gate, int ldg,
                                    int gate_parts, long long gate_part_stride, int gate_silu, const float* norm_w, float eps,
                                    hipStream_t stream) {
    if (B <= 0 || !delta_rows_ok(ld, parts, taps, state_stride, H, G, D, V)) return LLOGOS_BAD_ARGUMENT;
    if (z_parts < 1 || gate_parts < 1 || ldz < (channelwise ? H * D : H) || ldg < H * V || b_col < 0 || b_col + H > ld) return LLOGOS_BAD_ARGUMENT;
    const DeltaRows in{rows, ld, parts, (size_t)part_stride, conv, taps, 2 * G * D + H * V, state, (size_t)state_stride,
                       (size_t)H * D * V, slots, tok_pos, H, G, D, V};
    const DeltaGates gt{z, ldz, z_parts, (size_t)z_part_stride, dt_bias, a_log, channelwise, b_col};
    const bool vec = V % 4 == 0 && state_stride % 4 == 0 && (uintptr_t)state % 16 == 0;
    const int per = vec ? 4 : 1, threads = delta_step_threads(D, V, per);
    if (!threads) return LLOGOS_UNSUPPORTED;
    const int width = (V + per - 1) / per, P = threads / width, rpt = (D + P - 1) / P;
    const size_t smem = (size_t)(3 * D + 2 * V + width * per * (1 + 2 * P)) * sizeof(float);
    if (smem > 64 * 1024) return LLOGOS_UNSUPPORTED;
#define DS(VEC_, RPT_, NT, TAPS, TO) delta_step_kernel<VEC_, RPT_, NT, TAPS, TO><<<dim3(B, H), threads, smem, stream>>>((TO*)y, in, gt, \
        gate, ldg, gate_parts, (size_t)gate_part_stride, gate_silu, norm_w, eps)
#define DSV(NT, TAPS, TO) do { if (rpt <= 4) DS(4, 4, NT, TAPS, TO); else if (rpt <= 8) DS(4, 8, NT, TAPS, TO); else DS(4, 16, NT, TAPS, TO); } while (0)
#define DSR(TO) do { \
        if (!vec) { if (rpt <= 16) DS(1, 16, 1024, 16, TO); else DS(1, 64, 1024, 16, TO); } \
        else if (taps > 4 || threads > 512) DSV(1024, 16, TO); \
        else if (threads == 256) DSV(256, 4, TO); \
        else DSV(512, 4, TO); } while (0)
    if (y_dtype == DT_F32) DSR(float);
    else if (y_dtype == DT_BF16) DSR(bf16_t);
    else return LLOGOS_BAD_ARGUMENT;
#undef DSR
#undef DSV
#undef DS
    return LLOGOS_LAUNCH_CHECK();
}

// ---------------------------------------------------------------- longer steps: what the recurrence reads
// act [T][W]: q, k (unit vectors, q scaled) and v; logd: log2 of the decay, [T][H] or [T][H D]; beta [T][H].
// L lanes take a (token, unit): a head of q, of k or of v, the decays (all heads' together or a head's channels), beta.
template <int L>
__device__ __forceinline__ float delta_group_sum(float v) {
#pragma unroll
    for (int o = L / 2; o > 0; o >>= 1) v += __shfl_xor(v, o, kWave);
    return v;
}

template <int VEC, int L, int R>
__global__ __launch_bounds__(256) void delta_prepare_kernel(float* __restrict__ act, float* __restrict__ logd, float* __restrict__ beta,
                                                            DeltaRows in, DeltaGates gt, const int* __restrict__ tok_seq,
                                                            const int* __restrict__ cu) {
    const int t = blockIdx.x, lane = threadIdx.x % L;
    const int unit = blockIdx.y * (256 / L) + threadIdx.x / L;
    const int D = in.D, V = in.V, H = in.H, G = in.G;
    const int n_decay = gt.channelwise ? H : 1;
    const int seq = tok_seq[t], pos = in.tok_pos[t], before = t - cu[seq];
    const float* ring = in.state + (size_t)in.slots[seq] * in.state_stride + in.ring;
    if (unit >= 2 * G + H + n_decay + 1) return;
    auto conv = [&](int c, float (&out)[VEC]) {            // VEC neighbouring channels from c on
#pragma unroll
        for (int e = 0; e < VEC; ++e) out[e] = 0.f;
        for (int j = 0; j < in.taps; ++j) {                // the token's own row first
            const float* w = in.conv + (size_t)(in.taps - 1 - j) * in.W + c;
            if (VEC == 4) {
                float4 x = make_float4(0.f, 0.f, 0.f, 0.f);
                if (j <= before) {
                    const float* p = in.rows + (size_t)(t - j) * in.ld + c;
                    x = *reinterpret_cast<const float4*>(p);
                    for (int s = 1; s < in.parts; ++s) {
                        const float4 m = *reinterpret_cast<const float4*>(p + (size_t)s * in.part_stride);
                        x.x += m.x; x.y += m.y; x.z += m.z; x.w += m.w;
                    }
                } else if (pos >= j) {
                    x = *reinterpret_cast<const float4*>(ring + (size_t)((pos - j) % in.taps) * in.W + c);
                }
                const float4 wv = *reinterpret_cast<const float4*>(w);
                out[0] = fmaf(wv.x, x.x, out[0]);
                out[1 % VEC] = fmaf(wv.y, x.y, out[1 % VEC]);
                out[2 % VEC] = fmaf(wv.z, x.z, out[2 % VEC]);
                out[3 % VEC] = fmaf(wv.w, x.w, out[3 % VEC]);
            } else {
                out[0] = fmaf(w[0], delta_input(in, ring, t, pos, before, j, c), out[0]);
            }
        }
#pragma unroll
        for (int e = 0; e < VEC; ++e) out[e] = delta_silu(out[e]);
    };
    auto put = [&](float* p, const float (&x)[VEC], float f) {
        if (VEC == 4) *reinterpret_cast<float4*>(p) = make_float4(x[0] * f, x[1 % VEC] * f, x[2 % VEC] * f, x[3 % VEC] * f);
        else *p = x[0] * f;
    };
    float* row = act + (size_t)t * in.W;
    if (unit < 2 * G) {
        float x[R][VEC];
        float ss = 0.f;
#pragma unroll
        for (int r = 0; r < R; ++r) {
            const int d = (r * L + lane) * VEC;
            if (d < D) {
                conv(unit * D + d, x[r]);
#pragma unroll
                for (int e = 0; e < VEC; ++e) ss = fmaf(x[r][e], x[r][e], ss);
            }
        }
        float f = 1.0f / sqrtf(delta_group_sum<L>(ss) + 1e-6f);
        if (unit < G) f /= sqrtf((float)D);
#pragma unroll
        for (int r = 0; r < R; ++r) {
            const int d = (r * L + lane) * VEC;
            if (d < D) put(row + unit * D + d, x[r], f);
        }
    } else if (unit < 2 * G + H) {
        const int c0 = 2 * G * D + (unit - 2 * G) * V;
        for (int d = lane * VEC; d < V; d += L * VEC) {
            float x[VEC];
            conv(c0 + d, x);
            put(row + c0 + d, x, 1.0f);
        }
    } else if (unit < 2 * G + H + n_decay) {
        const int h0 = unit - 2 * G - H, n = gt.channelwise ? D : H, c0 = gt.channelwise ? h0 * D : 0;
        for (int i = lane; i < n; i += L) {
            const float z = delta_sum_parts(gt.z + (size_t)t * gt.ldz + c0 + i, gt.z_parts, gt.z_part_stride) + gt.dt_bias[c0 + i];
            logd[(size_t)t * (gt.channelwise ? H * D : H) + c0 + i] = delta_log_decay(z, gt.a_log[gt.channelwise ? h0 : i]);
        }
    } else {
        for (int i = lane; i < H; i += L)
            beta[(size_t)t * H + i] = delta_sigmoid(delta_sum_parts(in.rows + (size_t)t * in.ld + gt.b_col + i, in.parts, in.part_stride));
    }
}

// the ring behind a step of any length: the last min(taps, tokens) rows of every sequence.  Runs behind every reader.
__global__ void delta_ring_kernel(DeltaRows in, const int* __restrict__ cu) {
    const int seq = blockIdx.x, c = blockIdx.y * blockDim.x + threadIdx.x;
    if (c >= in.W) return;
    const int end = cu[seq + 1], count = end - cu[seq];
    float* ring = in.state + (size_t)in.slots[seq] * in.state_stride + in.ring;
    for (int back = 1; back <= min(in.taps, count); ++back) {
        const int t = end - back;
        ring[(size_t)(in.tok_pos[t] % in.taps) * in.W + c] = delta_sum_parts(in.rows + (size_t)t * in.ld + c, in.parts, in.part_stride);
    }
}

LLOGOS_EXPORT int llogos_delta_prepare(float* act, float* logd, float* beta, const float* rows, int ld, int parts, long long part_stride,
                                       const float* conv, int taps, float* state, long long state_stride, const int* slots,
                                       const int* tok_seq, const int* tok_pos, const int* cu, int T, int B, int H, int G, int D, int V,
                                       const float* z, int ldz, int z_parts, long long z_part_stride, const float* dt_bias,
                                       const float* a_log, int channelwise, int b_col, hipStream_t stream) {
    if (T <= 0 || B <= 0 || !cu || !delta_rows_ok(ld, parts, taps, state_stride, H, G, D, V)) return LLOGOS_BAD_ARGUMENT;
    if (z_parts < 1 || ldz < (channelwise ? H * D : H) || b_col < 0 || b_col + H > ld) return LLOGOS_BAD_ARGUMENT;
    const int W = 2 * G * D + H * V;
    const DeltaRows in{rows, ld, parts, (size_t)part_stride, conv, taps, W, state, (size_t)state_stride, (size_t)H * D * V, slots, tok_pos,
                       H, G, D, V};
    const DeltaGates gt{z, ldz, z_parts, (size_t)z_part_stride, dt_bias, a_log, channelwise, b_col};
    const int units = 2 * G + H + (channelwise ? H : 1) + 1;
    const bool vec = D % 4 == 0 && V % 4 == 0 && ld % 4 == 0 && part_stride % 4 == 0 && state_stride % 4 == 0 && ((size_t)H * D * V) % 4 == 0 &&
                     (uintptr_t)rows % 16 == 0 && (uintptr_t)state % 16 == 0 && (uintptr_t)conv % 16 == 0 && (uintptr_t)act % 16 == 0;
    if (vec) delta_prepare_kernel<4, 32, 2><<<dim3(T, (units + 7) / 8), 256, 0, stream>>>(act, logd, beta, in, gt, tok_seq, cu);
    else delta_prepare_kernel<1, 64, 4><<<dim3(T, (units + 3) / 4), 256, 0, stream>>>(act, logd, beta, in, gt, tok_seq, cu);
    delta_ring_kernel<<<dim3(B, (W + 255) / 256), 256, 0, stream>>>(in, cu);
    return LLOGOS_LAUNCH_CHECK();
}

// ---------------------------------------------------------------- longer steps: what does not depend on the state
// A chunk and head's workspace, in floats; fragments are 16 x 16 tiles, lane l's four values at 4 l (l & 15 a row of the
// first operand, 4 (l >> 4) .. + 3 its k), DTP tiles of key channels, VTN of value channels:
//   [2][DTP] -T K'   [2][DTP] q exp(b) - M K'   [DTP][2] (k exp(b_n - b))^T   [2][VTN] T V' (laid out as a result)   [16 DTP] exp(b_n)
__host__ __device__ __forceinline__ size_t delta_chunk_floats(int DTP, int VTN) { return (size_t)256 * (6 * DTP + 2 * VTN) + 16 * DTP; }

// A barrier for what the block's waves exchange through LDS alone: loads from memory that are on their way, and stores,
// are not waited for (__syncthreads waits for all of them, and with them for everything asked for ahead).
__device__ __forceinline__ void delta_lds_barrier() {
    asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");
    __builtin_amdgcn_s_barrier();
    asm volatile("" ::: "memory");
}

__device__ __forceinline__ dl4 delta_mfma4(dl4 a, dl4 b, dl4 acc) {
#pragma unroll
    for (int e = 0; e < 4; ++e) acc = __builtin_amdgcn_mfma_f32_16x16x4f32(a[e], b[e], acc, 0, 0, 0);
    return acc;
}
__device__ __forceinline__ dl4 delta_ld4(const float* p) { return *reinterpret_cast<const dl4*>(p); }
__device__ __forceinline__ dl4 delta_exp2(dl4 x) { return dl4{delta_exp2(x[0]), delta_exp2(x[1]), delta_exp2(x[2]), delta_exp2(x[3])}; }

// Which chunk is this: its sequence, first token and number of tokens (false: beyond the last).
__device__ __forceinline__ bool delta_find_chunk(const int* __restrict__ cu, int B, int chunk, int& first, int& n) {
    for (int b = 0; b < B; ++b) {
        const int len = cu[b + 1] - cu[b], chunks = (len + kDeltaChunk - 1) / kDeltaChunk;
        if (chunk < chunks) {
            first = cu[b] + chunk * kDeltaChunk;
            n = min(kDeltaChunk, len - chunk * kDeltaChunk);
            return true;
        }
        chunk -= chunks;
    }
    return false;
}

// LDS: q, k [32][16 DTP + 4], with a decay a channel the sums of logarithms in the same shape, A, P, T, M [32][36]
__host__ __device__ __forceinline__ int delta_chunk_lds(int DTP, bool channelwise) {
    return (channelwise ? 3 : 2) * kDeltaChunk * (16 * DTP + kDeltaPad) + 4 * kDeltaChunk * kDeltaCP;
}

// grid (chunks, heads), four waves.
template <bool CHANNELWISE>
__global__ __launch_bounds__(256) void delta_chunk_kernel(float* __restrict__ ws, float* __restrict__ o, const float* __restrict__ act,
                                                          const float* __restrict__ logd, const float* __restrict__ beta,
                                                          const int* __restrict__ cu, int B, int H, int G, int D, int V, int DTP, int VTN,
                                                          int vec) {
    constexpr int C = kDeltaChunk, CP = kDeltaCP;
    extern __shared__ __attribute__((aligned(16))) float lds[];
    const int DP = 16 * DTP + kDeltaPad;
    float* sQ = lds;
    float* sK = sQ + C * DP;
    float* sB = sK + C * DP;                               // sums of logarithms within each run of 16 tokens, a channel (or unused)
    float* sA = sB + (CHANNELWISE ? C * DP : 0);
    float* sP = sA + C * CP;
    float* sT = sP + C * CP;
    float* sM = sT + C * CP;
    __shared__ __attribute__((aligned(16))) float s_beta[C], s_b[C];
    int first, n;
    if (!delta_find_chunk(cu, B, blockIdx.x, first, n)) return;
    const int head = blockIdx.y, kvh = head / (H / G), W = 2 * G * D + H * V;
    const int tid = threadIdx.x, lane = tid & (kWave - 1), wave = tid / kWave, c = lane & 15, g = lane >> 4;
    float* out = ws + ((size_t)blockIdx.x * H + head) * delta_chunk_floats(DTP, VTN);

    if (tid < C) s_beta[tid] = tid < n ? beta[(size_t)(first + tid) * H + head] : 0.f;
#pragma unroll 4
    for (int e = tid; e < C * 4 * DTP; e += 256) {
        const int j = e / (4 * DTP), d = 4 * (e % (4 * DTP));
        dl4 q = {0.f, 0.f, 0.f, 0.f}, k = q;
        if (j < n && d < D) {
            const float* p = act + (size_t)(first + j) * W + kvh * D + d;
            if (vec) {
                q = delta_ld4(p);
                k = delta_ld4(p + G * D);
            } else {
#pragma unroll
                for (int i = 0; i < 4; ++i)
                    if (d + i < D) { q[i] = p[i]; k[i] = p[G * D + i]; }
            }
        }
        *reinterpret_cast<dl4*>(sQ + j * DP + d) = q;
        *reinterpret_cast<dl4*>(sK + j * DP + d) = k;
    }
    if (CHANNELWISE) {
        for (int d = tid; d < 16 * DTP; d += 256) {
            float x[C];
#pragma unroll
            for (int j = 0; j < C; ++j) x[j] = (j < n && d < D) ? logd[(size_t)(first + j) * H * D + head * D + d] : 0.f;
            float run = 0.f;
#pragma unroll
            for (int j = 0; j < C; ++j) {
                run = (j == 16 ? 0.f : run) + x[j];
                sB[j * DP + d] = run;
            }
        }
    } else if (wave == 0) {
        // lanes 0..15 and 16..31 each sum their own run
        float x = lane < n && lane < C ? logd[(size_t)(first + lane) * H + head] : 0.f;
#pragma unroll
        for (int s = 1; s < 16; s <<= 1) {
            const float y = __shfl_up(x, s, 16);
            if (c >= s) x += y;
        }
        if (lane < C) s_b[lane] = x;
    }
    delta_lds_barrier();
    // the logarithm's sum within row j's run of 16, channel d .. d + 3
    auto rel4 = [&](int j, int d) {
        if (CHANNELWISE) return delta_ld4(sB + j * DP + d);
        const float b = s_b[j];
        return dl4{b, b, b, b};
    };
    auto rel = [&](int j, int d) { return CHANNELWISE ? sB[j * DP + d] : s_b[j]; };

    // ---- A and P, tiles (0, 0), (1, 0), (1, 1)
    if (!CHANNELWISE) {
        if (wave < 3) {
            const int it = wave > 0 ? 1 : 0, jt = wave > 1 ? 1 : 0;
            dl4 kk = {0.f, 0.f, 0.f, 0.f}, qk = kk;
            for (int dt = 0; dt < DTP; ++dt) {
                const dl4 kj = delta_ld4(sK + (16 * jt + c) * DP + 16 * dt + 4 * g);
                const dl4 ki = delta_ld4(sK + (16 * it + c) * DP + 16 * dt + 4 * g);
                const dl4 qi = delta_ld4(sQ + (16 * it + c) * DP + 16 * dt + 4 * g);
                kk = delta_mfma4(ki, kj, kk);
                qk = delta_mfma4(qi, kj, qk);
            }
#pragma unroll
            for (int r = 0; r < 4; ++r) {
                const int i = 16 * it + 4 * g + r, j = 16 * jt + c;
                const float f = j <= i ? delta_exp2(it == jt ? s_b[i] - s_b[j] : s_b[i] + (s_b[15] - s_b[j])) : 0.f;
                sA[i * CP + j] = j < i ? s_beta[i] * kk[r] * f : 0.f;
                sP[i * CP + j] = qk[r] * f;
            }
        }
    } else {
        // the tiles on the diagonal pair by pair: the decays' quotients differ from channel to channel.  A wave takes a tile
        // and half of the channels, a lane 2 x 2 pairs; the halves meet in LDS.
        {
            const int it = wave >> 1, half = wave & 1, i0 = 16 * it + 2 * (lane >> 3), j0 = 16 * it + 2 * (lane & 7);
            const int mid = 8 * DTP, d_end = half ? min(16 * DTP, (D + 3) & ~3) : min(mid, (D + 3) & ~3);        // (channels behind D hold zeros)
            float kk[2][2] = {{0.f, 0.f}, {0.f, 0.f}}, qk[2][2] = {{0.f, 0.f}, {0.f, 0.f}};
            if (j0 <= i0 + 1) {
                for (int d = half ? mid : 0; d < d_end; d += 4) {
                    dl4 ki[2], qi[2], bi[2], kj[2], bj[2];
#pragma unroll
                    for (int a = 0; a < 2; ++a) {
                        ki[a] = delta_ld4(sK + (i0 + a) * DP + d);
                        qi[a] = delta_ld4(sQ + (i0 + a) * DP + d);
                        bi[a] = delta_ld4(sB + (i0 + a) * DP + d);
                        kj[a] = delta_ld4(sK + (j0 + a) * DP + d);
                        bj[a] = delta_ld4(sB + (j0 + a) * DP + d);
                    }
#pragma unroll
                    for (int a = 0; a < 2; ++a)
#pragma unroll
                        for (int b = 0; b < 2; ++b) {
                            // (a pair above the diagonal is not used; its exponent would be positive)
                            const dl4 x = kj[b] * delta_exp2(j0 + b <= i0 + a ? bi[a] - bj[b] : dl4{0.f, 0.f, 0.f, 0.f});
#pragma unroll
                            for (int e = 0; e < 4; ++e) {
                                kk[a][b] = fmaf(ki[a][e], x[e], kk[a][b]);
                                qk[a][b] = fmaf(qi[a][e], x[e], qk[a][b]);
                            }
                        }
                }
            }
            float* hA = sT + it * 16 * CP;                 // (T and M are not there yet)
            float* hP = sM + it * 16 * CP;
            if (half) {
#pragma unroll
                for (int a = 0; a < 2; ++a)
#pragma unroll
                    for (int b = 0; b < 2; ++b) {
                        hA[(i0 + a - 16 * it) * CP + j0 + b - 16 * it] = kk[a][b];
                        hP[(i0 + a - 16 * it) * CP + j0 + b - 16 * it] = qk[a][b];
                    }
            }
            delta_lds_barrier();
            if (!half) {
#pragma unroll
                for (int a = 0; a < 2; ++a)
#pragma unroll
                    for (int b = 0; b < 2; ++b) {
                        const int i = i0 + a, j = j0 + b;
                        sA[i * CP + j] = j < i ? s_beta[i] * (kk[a][b] + hA[(i - 16 * it) * CP + j - 16 * it]) : 0.f;
                        sP[i * CP + j] = j <= i ? qk[a][b] + hP[(i - 16 * it) * CP + j - 16 * it] : 0.f;
                    }
            }
        }
        if (wave == 1) {                                   // (the waves of the halves have less to do at the end)
            dl4 kk = {0.f, 0.f, 0.f, 0.f}, qk = kk;
            for (int dt = 0; dt < DTP; ++dt) {
                const int d = 16 * dt + 4 * g;
                const dl4 kj = delta_ld4(sK + c * DP + d) * delta_exp2(rel4(15, d) - rel4(c, d));
                const dl4 bi = delta_exp2(rel4(16 + c, d));
                kk = delta_mfma4(delta_ld4(sK + (16 + c) * DP + d) * bi, kj, kk);
                qk = delta_mfma4(delta_ld4(sQ + (16 + c) * DP + d) * bi, kj, qk);
            }
#pragma unroll
            for (int r = 0; r < 4; ++r) {
                const int i = 16 + 4 * g + r;
                sA[i * CP + c] = s_beta[i] * kk[r];
                sP[i * CP + c] = qk[r];
            }
        }
    }
    delta_lds_barrier();
    // ---- T = (I + A)^-1: the diagonal tiles column by column, the tile below from them
    if (wave < 2) {
        const float* a = sA + 16 * wave * CP + 16 * wave;
        float x[16];
#pragma unroll
        for (int i = 0; i < 16; ++i) {
            float s = i == c ? 1.f : 0.f;
#pragma unroll
            for (int j = 0; j < i; ++j) s = fmaf(-a[i * CP + j], x[j], s);
            x[i] = s;
        }
        if (g == 0) {
#pragma unroll
            for (int i = 0; i < 16; ++i) sT[(16 * wave + i) * CP + 16 * wave + c] = x[i];
        }
    }
    delta_lds_barrier();
    auto column4 = [&](const float* m, int r0, int col) {  // rows r0 .. r0 + 3 of a column of a [32][36] matrix
        return dl4{m[r0 * CP + col], m[(r0 + 1) * CP + col], m[(r0 + 2) * CP + col], m[(r0 + 3) * CP + col]};
    };
    if (wave == 0) {
        dl4 z = {0.f, 0.f, 0.f, 0.f}, t = z;
        z = delta_mfma4(delta_ld4(sA + (16 + c) * CP + 4 * g), column4(sT, 4 * g, c), z);
        t = delta_mfma4(delta_ld4(sT + (16 + c) * CP + 16 + 4 * g), z, t);
#pragma unroll
        for (int r = 0; r < 4; ++r) sT[(16 + 4 * g + r) * CP + c] = -t[r];
    }
    delta_lds_barrier();
    // ---- M = P T
    if (wave < 3) {
        const int it = wave > 0 ? 1 : 0, jt = wave > 1 ? 1 : 0;
        dl4 m = {0.f, 0.f, 0.f, 0.f};
        for (int kt = jt; kt <= it; ++kt)
            m = delta_mfma4(delta_ld4(sP + (16 * it + c) * CP + 16 * kt + 4 * g), column4(sT, 16 * kt + 4 * g, 16 * jt + c), m);
#pragma unroll
        for (int r = 0; r < 4; ++r) sM[(16 * it + 4 * g + r) * CP + 16 * jt + c] = m[r];
    }
    delta_lds_barrier();
    // ---- the products with K' and V'
    const dl4 t00 = delta_ld4(sT + c * CP + 4 * g), t10 = delta_ld4(sT + (16 + c) * CP + 4 * g), t11 = delta_ld4(sT + (16 + c) * CP + 16 + 4 * g);
    const dl4 m00 = delta_ld4(sM + c * CP + 4 * g), m10 = delta_ld4(sM + (16 + c) * CP + 4 * g), m11 = delta_ld4(sM + (16 + c) * CP + 16 + 4 * g);
    const dl4 be[2] = {delta_ld4(s_beta + 4 * g), delta_ld4(s_beta + 16 + 4 * g)};
    const dl4 zero = {0.f, 0.f, 0.f, 0.f};
    for (int dt = wave; dt < DTP; dt += 4) {
        const int d = 16 * dt + c;
        const float b15 = rel(15, d), b31 = rel(31, d);
        dl4 kb[2], ke[2];
#pragma unroll
        for (int jt = 0; jt < 2; ++jt) {
#pragma unroll
            for (int e = 0; e < 4; ++e) {
                const int j = 16 * jt + 4 * g + e;
                const float k = sK[j * DP + d], b = rel(j, d);
                kb[jt][e] = be[jt][e] * k * delta_exp2(jt ? b + b15 : b);
                ke[jt][e] = k * delta_exp2(jt ? b31 - b : (b15 - b) + b31);
            }
        }
        dl4 w0 = delta_mfma4(kb[0], t00, zero);
        dl4 w1 = delta_mfma4(kb[1], t11, delta_mfma4(kb[0], t10, zero));
        dl4 q0 = delta_mfma4(kb[0], m00, zero);
        dl4 q1 = delta_mfma4(kb[1], m11, delta_mfma4(kb[0], m10, zero));
        const int dq = 16 * dt + 4 * g;
        const dl4 qd0 = delta_ld4(sQ + c * DP + dq) * delta_exp2(rel4(c, dq));
        const dl4 qd1 = delta_ld4(sQ + (16 + c) * DP + dq) * delta_exp2(rel4(16 + c, dq) + rel4(15, dq));
        dl4* f = reinterpret_cast<dl4*>(out);
        f[(size_t)dt * 64 + lane] = -w0;
        f[(size_t)(DTP + dt) * 64 + lane] = -w1;
        f[(size_t)(2 * DTP + dt) * 64 + lane] = qd0 - q0;
        f[(size_t)(3 * DTP + dt) * 64 + lane] = qd1 - q1;
        f[(size_t)(4 * DTP + 2 * dt) * 64 + lane] = ke[0];
        f[(size_t)(4 * DTP + 2 * dt + 1) * 64 + lane] = ke[1];
        if (g == 0) out[(size_t)256 * (6 * DTP + 2 * VTN) + d] = delta_exp2(b15 + b31);
    }
    for (int vt = wave; vt < VTN; vt += 4) {
        const int col = 16 * vt + c;
        dl4 vb[2];
#pragma unroll
        for (int jt = 0; jt < 2; ++jt) {
#pragma unroll
            for (int e = 0; e < 4; ++e) {
                const int j = 16 * jt + 4 * g + e;
                vb[jt][e] = (j < n && col < V) ? be[jt][e] * act[(size_t)(first + j) * W + 2 * G * D + head * V + col] : 0.f;
            }
        }
        const dl4 y0 = delta_mfma4(t00, vb[0], zero);
        const dl4 y1 = delta_mfma4(t11, vb[1], delta_mfma4(t10, vb[0], zero));
        const dl4 o0 = delta_mfma4(m00, vb[0], zero);
        const dl4 o1 = delta_mfma4(m11, vb[1], delta_mfma4(m10, vb[0], zero));
        dl4* f = reinterpret_cast<dl4*>(out + (size_t)256 * 6 * DTP);
        f[(size_t)vt * 64 + lane] = y0;
        f[(size_t)(VTN + vt) * 64 + lane] = y1;
        if (col < V) {
#pragma unroll
            for (int r = 0; r < 4; ++r) {
                const int i = 4 * g + r;
                if (i < n) o[((size_t)(first + i) * H + head) * V + col] = o0[r];
                if (16 + i < n) o[((size_t)(first + 16 + i) * H + head) * V + col] = o1[r];
            }
        }
    }
}

// ---------------------------------------------------------------- longer steps: the state from chunk to chunk
// grid (sequences x heads, tiles of 16 columns); NW waves, each with DTW tiles of 16 key channels of those columns of S in
// registers, laid out as a product's result, which is also the operand its next use wants.  A chunk: every wave's share of
// -T K' S and (q exp(b) - M K') S, the waves' shares added through LDS (two buffers in turn: one barrier a chunk), then
// the update of its own tiles from all of U.  The next chunk's fragments are on their way meanwhile.
template <int NW, int DTW>
struct DeltaFrags {
    dl4 w[2][DTW], q[2][DTW], k[DTW][2], y[2], gain[DTW];
    float o[NW == 1 ? 2 : 1][4];               // what the chunk alone gives of o, for the tile (or both) that this wave finishes
};

template <int NW, int DTW>
__global__ __launch_bounds__(NW * kWave) void delta_scan_kernel(float* __restrict__ o, const float* __restrict__ ws, float* __restrict__ state,
                                                                size_t state_stride, const int* __restrict__ slots,
                                                                const int* __restrict__ cu, int H, int D, int V, int VTN) {
    constexpr int C = kDeltaChunk, DTP = NW * DTW;
    __shared__ dl4 red[2][NW][4][kWave];
    const int seq = blockIdx.x / H, head = blockIdx.x % H, vt = blockIdx.y;
    const int tid = threadIdx.x, lane = tid & (kWave - 1), wave = tid / kWave, c = lane & 15, g = lane >> 4;
    const int first = cu[seq], count = cu[seq + 1] - first, col = 16 * vt + c;
    int chunk0 = 0;
    for (int b = 0; b < seq; ++b) chunk0 += (cu[b + 1] - cu[b] + C - 1) / C;
    const int chunks = (count + C - 1) / C;
    const size_t stride = delta_chunk_floats(DTP, VTN);
    const float* mine = ws + ((size_t)chunk0 * H + head) * stride;
    float* S = state + (size_t)slots[seq] * state_stride + (size_t)head * D * V;
    // the tile of o that this wave finishes (waves 0 and 1, or wave 0 both)
    const int o_tiles = NW == 1 ? 2 : (wave < 2 ? 1 : 0);

    dl4 s[DTW];
#pragma unroll
    for (int dt = 0; dt < DTW; ++dt)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
            const int d = 16 * (wave * DTW + dt) + 4 * g + r;
            s[dt][r] = (d < D && col < V) ? S[(size_t)d * V + col] : 0.f;
        }
    auto fetch = [&](DeltaFrags<NW, DTW>& f, int ch) {
        const float* p = mine + (size_t)ch * H * stride;
        const dl4* t = reinterpret_cast<const dl4*>(p);
#pragma unroll
        for (int dt = 0; dt < DTW; ++dt) {
            const int d = wave * DTW + dt;
#pragma unroll
            for (int it = 0; it < 2; ++it) {
                f.w[it][dt] = t[(size_t)(it * DTP + d) * 64 + lane];
                f.q[it][dt] = t[(size_t)((2 + it) * DTP + d) * 64 + lane];
                f.k[dt][it] = t[(size_t)(4 * DTP + 2 * d + it) * 64 + lane];
            }
            f.gain[dt] = delta_ld4(p + (size_t)256 * (6 * DTP + 2 * VTN) + 16 * d + 4 * g);
        }
#pragma unroll
        for (int it = 0; it < 2; ++it) f.y[it] = t[(size_t)(6 * DTP + it * VTN + vt) * 64 + lane];
#pragma unroll
        for (int x = 0; x < (NW == 1 ? 2 : 1); ++x)
#pragma unroll
            for (int r = 0; r < 4; ++r) {
                // (what lies outside is read from the nearest place inside and never stored)
                const int i = min(C * ch + 16 * (NW == 1 ? x : min(wave, 1)) + 4 * g + r, count - 1);
                f.o[x][r] = o[((size_t)(first + i) * H + head) * V + min(col, V - 1)];
            }
    };
    // A chunk's o is stored while a later one is worked on, in front of what is asked for then: whoever waits for those loads
    // (they are counted in order) waits for no store that has just begun.
    float done[NW == 1 ? 2 : 1][4];
    auto put = [&](int ch) {
        if (o_tiles == 0 || col >= V) return;
#pragma unroll
        for (int x = 0; x < (NW == 1 ? 2 : 1); ++x) {
            const int i = C * ch + 16 * (NW == 1 ? x : wave) + 4 * g;
            float* p = o + ((size_t)(first + i) * H + head) * V + col;
            if (C * ch + C <= count) {
#pragma unroll
                for (int r = 0; r < 4; ++r) p[(size_t)r * H * V] = done[x][r];
            } else {
#pragma unroll
                for (int r = 0; r < 4; ++r)
                    if (i + r < count) p[(size_t)r * H * V] = done[x][r];
            }
        }
    };
    auto work = [&](const DeltaFrags<NW, DTW>& f, int ch) {
        dl4 u[2], q[2];
#pragma unroll
        for (int it = 0; it < 2; ++it) u[it] = q[it] = dl4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int dt = 0; dt < DTW; ++dt) {
            // (four chains in turn: a product's result is not waited for by the next)
#pragma unroll
            for (int e = 0; e < 4; ++e) {
                const float b = s[dt][e];
                u[0] = __builtin_amdgcn_mfma_f32_16x16x4f32(f.w[0][dt][e], b, u[0], 0, 0, 0);
                u[1] = __builtin_amdgcn_mfma_f32_16x16x4f32(f.w[1][dt][e], b, u[1], 0, 0, 0);
                q[0] = __builtin_amdgcn_mfma_f32_16x16x4f32(f.q[0][dt][e], b, q[0], 0, 0, 0);
                q[1] = __builtin_amdgcn_mfma_f32_16x16x4f32(f.q[1][dt][e], b, q[1], 0, 0, 0);
            }
        }
        if (NW > 1) {
            dl4 (*buf)[4][kWave] = red[ch & 1];
            buf[wave][0][lane] = u[0];
            buf[wave][1][lane] = u[1];
            buf[wave][2][lane] = q[0];
            buf[wave][3][lane] = q[1];
            delta_lds_barrier();
#pragma unroll
            for (int it = 0; it < 2; ++it) {
                u[it] = buf[0][it][lane];
#pragma unroll
                for (int w = 1; w < NW; ++w) u[it] += buf[w][it][lane];
            }
            if (wave < 2) {
                q[0] = buf[0][2 + wave][lane];
#pragma unroll
                for (int w = 1; w < NW; ++w) q[0] += buf[w][2 + wave][lane];
            }
        }
#pragma unroll
        for (int it = 0; it < 2; ++it) u[it] += f.y[it];
#pragma unroll
        for (int x = 0; x < (NW == 1 ? 2 : 1); ++x)
#pragma unroll
            for (int r = 0; r < 4; ++r) done[x][r] = f.o[x][r] + q[x][r];
#pragma unroll
        for (int dt = 0; dt < DTW; ++dt) s[dt] *= f.gain[dt];
#pragma unroll
        for (int jt = 0; jt < 2; ++jt)
#pragma unroll
            for (int e = 0; e < 4; ++e)
#pragma unroll
                for (int dt = 0; dt < DTW; ++dt)
                    s[dt] = __builtin_amdgcn_mfma_f32_16x16x4f32(f.k[dt][jt][e], u[jt][e], s[dt], 0, 0, 0);
    };
    // AHEAD sets of fragments in turn: a chunk's are asked for AHEAD - 1 chunks before they are worked on
    constexpr int AHEAD = DTW <= 2 ? 3 : 2;
    DeltaFrags<NW, DTW> set[AHEAD];
#pragma unroll
    for (int k = 0; k < AHEAD; ++k) fetch(set[k], min(k, chunks - 1));
    int ch0 = 0;
    for (; ch0 + AHEAD <= chunks; ch0 += AHEAD) {          // (no branch around the loads: how many are newer is known where one is waited for)
#pragma unroll
        for (int k = 0; k < AHEAD; ++k) {
            __builtin_amdgcn_sched_barrier(0);
            work(set[k], ch0 + k);
            put(ch0 + k);
            fetch(set[k], min(ch0 + k + AHEAD, chunks - 1));
            __builtin_amdgcn_sched_barrier(0);              // (the loads stay where they are)
        }
    }
#pragma unroll
    for (int k = 0; k < AHEAD - 1; ++k)
        if (ch0 + k < chunks) {
            work(set[k], ch0 + k);
            put(ch0 + k);
        }
#pragma unroll
    for (int dt = 0; dt < DTW; ++dt)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
            const int d = 16 * (wave * DTW + dt) + 4 * g + r;
            if (d < D && col < V) S[(size_t)d * V + col] = s[dt][r];
        }
}

// tiles of 16 key channels with which the two kernels work: the waves of a block share them out evenly
static int delta_tiles(int D) {
    const int dt = (D + 15) / 16;
    return dt <= 2 ? dt : (dt + 3) / 4 * 4;
}

// floats of workspace for a step of so many chunks (each sequence's tokens in chunks of 32)
LLOGOS_EXPORT long long llogos_delta_workspace(int chunks, int H, int D, int V) {
    if (chunks <= 0 || H <= 0 || D <= 0 || V <= 0) return 0;
    return (long long)chunks * H * (long long)delta_chunk_floats(delta_tiles(D), (V + 15) / 16);
}

// o [T][H V] from act, logd and beta (llogos_delta_prepare) and the state, which is brought up to date.
LLOGOS_EXPORT int llogos_delta_scan(float* o, const float* act, const float* logd, const float* beta, float* ws, long long ws_floats,
                                    float* state, long long state_stride, const int* slots, const int* cu, int B, int chunks, int H,
                                    int G, int D, int V, int channelwise, hipStream_t stream) {
    if (B <= 0 || chunks <= 0 || H <= 0 || G <= 0 || H % G || D <= 0 || V <= 0 || D > kDeltaMaxDim || V > kDeltaMaxV || !cu) return LLOGOS_BAD_ARGUMENT;
    if (state_stride < (long long)H * D * V || ws_floats < llogos_delta_workspace(chunks, H, D, V) || (uintptr_t)ws % 16) return LLOGOS_BAD_ARGUMENT;
    const int DTP = delta_tiles(D), VTN = (V + 15) / 16, W = 2 * G * D + H * V;
    const int vec = D % 4 == 0 && W % 4 == 0 && (uintptr_t)act % 16 == 0 ? 1 : 0;
    const int smem = delta_chunk_lds(DTP, channelwise) * (int)sizeof(float);
#define DCK(CW) do { \
        if (smem > 48 * 1024) { \
            hipError_t e = hipFuncSetAttribute((const void*)delta_chunk_kernel<CW>, hipFuncAttributeMaxDynamicSharedMemorySize, smem); \
            if (e != hipSuccess) return (int)e; \
        } \
        delta_chunk_kernel<CW><<<dim3(chunks, H), 256, smem, stream>>>(ws, o, act, logd, beta, cu, B, H, G, D, V, DTP, VTN, vec); } while (0)
    if (channelwise) DCK(true); else DCK(false);
#undef DCK
    const dim3 grid(B * H, VTN);
#define DSC(NW, DTW) delta_scan_kernel<NW, DTW><<<grid, NW * kWave, 0, stream>>>(o, ws, state, (size_t)state_stride, slots, cu, H, D, V, VTN)
    if (DTP == 1) DSC(1, 1); else if (DTP == 2) DSC(2, 1); else if (DTP == 4) DSC(4, 1); else if (DTP == 8) DSC(4, 2);
    else if (DTP == 12) DSC(4, 3); else DSC(4, 4);
#undef DSC
    return LLOGOS_LAUNCH_CHECK();
}

// ---------------------------------------------------------------- longer steps: norm over a head, weight, gate
// One wave a (token, head).
template <typename TO>
__global__ __launch_bounds__(256) void delta_out_kernel(TO* __restrict__ y, const float* __restrict__ o, const float* __restrict__ gate,
                                                        int ldg, int parts, size_t part_stride, int gate_silu,
                                                        const float* __restrict__ w, float eps, int H, int V, int items) {
    const int item = blockIdx.x * 4 + threadIdx.x / kWave, lane = threadIdx.x & (kWave - 1);
    if (item >= items) return;
    const int t = item / H, head = item % H;
    const float* row = o + (size_t)item * V;
    const float* z = gate + (size_t)t * ldg + (size_t)head * V;
    float ss = 0.f;
    for (int i = lane; i < V; i += kWave) ss = fmaf(row[i], row[i], ss);
    const float inv = 1.0f / sqrtf(wave_sum(ss) / (float)V + eps);
    for (int i = lane; i < V; i += kWave) {
        const float g = delta_sum_parts(z + i, parts, part_stride);
        store_f32(y + (size_t)item * V + i, row[i] * inv * w[i] * (gate_silu ? delta_silu(g) : delta_sigmoid(g)));
    }
}

LLOGOS_EXPORT int llogos_delta_out(void* y, int y_dtype, const float* o, const float* gate, int ldg, int parts, long long part_stride,
                                   int gate_silu, const float* w, float eps, int T, int H, int V, hipStream_t stream) {
    if (T <= 0 || H <= 0 || V <= 0 || parts < 1 || ldg < H * V) return LLOGOS_BAD_ARGUMENT;
    const int items = T * H, blocks = (items + 3) / 4;
    if (y_dtype == DT_F32) delta_out_kernel<float><<<blocks, 256, 0, stream>>>((float*)y, o, gate, ldg, parts, (size_t)part_stride, gate_silu, w, eps, H, V, items);
    else if (y_dtype == DT_BF16) delta_out_kernel<bf16_t><<<blocks, 256, 0, stream>>>((bf16_t*)y, o, gate, ldg, parts, (size_t)part_stride, gate_silu, w, eps, H, V, items);
    else return LLOGOS_BAD_ARGUMENT;
    return LLOGOS_LAUNCH_CHECK();
}
