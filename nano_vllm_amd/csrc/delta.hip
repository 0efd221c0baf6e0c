// The gated delta rule with a decay per key channel, after its projections: a linear attention over a state
// of fixed size per request that forgets channel by channel and, at every token, is corrected towards the value
// its key should read out.
//
//   proj [T, 2 G D + H DV + H] = [q | k | v | b]        elements; G query/key heads of D, H value heads of DV
//   q, k, v <- silu(sum over the last `taps` tokens of w[c][j] * input[c])      per channel c, no bias; the inputs
//              before a portion come from the request's kept inputs (conv_state), zeros before its start
//   q <- q / sqrt(sum(q^2) + 1e-6) * D^-1/2,  k <- k / sqrt(sum(k^2) + 1e-6)    per head
//   beta = sigmoid(b)                                                            per value head
//   a = exp(-exp(a_log[h]) * softplus(decay_in[h][d] + dt_bias[h][d]))          per value head and key channel
//   per value head h, with its query/key head h / (H / G), S [D, DV]:
//       S <- diag(a) S;   u = beta (v - S^T k);   S <- S + k u^T;   o = S^T q
//   y = o / sqrt(mean(o^2) + eps) * norm_w * sigmoid(gate_in)                   per head, norm_w [DV]
//
// With one decay per head (nva_head_delta) a is one number for all key channels of a value head, computed from one
// input per head; beta's and the decay's inputs come as floats from a product of their own, rates [T, 2 H] = [b | a]; the
// gate is silu(gate_in) and gate_in the columns of proj behind [q | k | v].
//
// Everything after the projections is float whatever the element type (the convolutions' sums, the unit norms,
// softplus and the exponentials by the accurate routines, the state, the read-out, the norm and the gate); y is
// rounded once.  A token's sums run in an order that neither the portion's cut nor the batch changes: the
// recurrence goes token by token, 8 or 16 lanes holding one column of S in registers.
//
//   delta_prepare     one workgroup per (token, head of q, k or v): the convolutions, unit norms, beta and the decay,
//                     written as floats
//   delta_keep        the request's new kept inputs (its last taps - 1), after delta_prepare has read the old ones
//   delta_scan        four waves per (request, head, 16 or 32 columns of S), 16 or 8 lanes a column: the recurrence over the
//                     portion's tokens, the tokens' q, k, a and beta staged in LDS a batch at a time in two buffers,
//                     v asked for a batch ahead
//   delta_finish      one wave per (token, head): the norm and the gate
//
// With one decay per head two more ways run the same rule:
//   delta_single      a request that brings one token: everything above for one (request, value head) in one workgroup
//   delta_block_*     portions of many tokens, in blocks of 64 on the matrix cores (float products).  With G_i the sum of
//                     the logarithms of the decays up to token i of a block, S_0 the state before the block, and
//                     A_ij = beta_i exp(G_i - G_j) k_i.k_j for j < i, the writes of the block are
//                         (I + A) u = beta v - beta exp(G) k^T S_0      (row i: beta_i v_i - beta_i exp(G_i) S_0^T k_i)
//                     so u = U - W S_0 with (I + A) U = beta v and (I + A) W = beta exp(G) k, both by forward
//                     substitution; then o_i = exp(G_i) S_0^T q_i + sum over j <= i of P_ij u_j with P_ij = exp(G_i - G_j)
//                     q_i.k_j, and the state behind the block is exp(G_63) S_0 + sum over j of exp(G_63 - G_j) k_j u_j^T.
//     delta_block_prepare   the convolutions, unit norms, beta and log decays, 16 tokens of a head to a workgroup
//     delta_block_solve     a workgroup per (block, head): A and P by products; U and W by substitution in blocks of 16 rows,
//                           the diagonal blocks of I + A inverted row by row, everything else products
//     delta_block_scan      a workgroup per (portion, head, 16 columns of S): the blocks one after the other
#include "common.h"

typedef __attribute__((ext_vector_type(4))) float delta_f32x4;

#define DELTA_MAX_TAPS 16
#define DELTA_BATCH 8            // tokens whose q, k and a lie in LDS at a time
#define DELTA_THREADS 256        // of the recurrence's workgroup: four waves
#define DELTA_MAX_DIM 256        // key channels of a head at most
#define DELTA_PREPARE_THREADS 128
#define DELTA_BLOCK 64            // tokens of a block of the matrix-core form
#define DELTA_SINGLE_THREADS 512

// One workgroup per (token, unit); a unit is a query head, a key head, or a value head with its decays and beta.
// Rows of qn, kn and decay are DP = dim rounded up to 4 floats apart, the padding zero.
// Entry i of a token's rates [b | a], which may be left as partial sums of their product.
struct DeltaRates {
    const float* sums;               // [splits][tokens][2 heads]
    int splits;
    int64_t split_stride;
};
__device__ __forceinline__ float delta_rate(const DeltaRates& r, int64_t t, int heads, int i) {
    float v = 0.f;
    for (int s = 0; s < r.splits; ++s) v += r.sums[s * r.split_stride + t * (2 * heads) + i];
    return v;
}
__device__ __forceinline__ float delta_softplus(float z) { return z > 20.f ? z : log1pf(expf(z)); }

// HEAD: one decay per value head; `decay` [tokens, heads] then receives its logarithm.  t0: the first token of the launch.
template <typename T, bool HEAD>
__global__ void __launch_bounds__(DELTA_PREPARE_THREADS)
delta_prepare_kernel(const T* __restrict__ proj, int64_t stride, const float* __restrict__ decay_in, DeltaRates rates, int64_t t0,
                     const T* __restrict__ conv_w, const float* __restrict__ dt_bias, const float* __restrict__ a_log,
                     const float* __restrict__ conv_state, const int32_t* __restrict__ token_seq,
                     const int32_t* __restrict__ cu_seqlens_q, const int32_t* __restrict__ seq_starts,
                     const int32_t* __restrict__ state_slots, int heads, int kv_heads, int dim, int vdim, int taps,
                     float* __restrict__ qn, float* __restrict__ kn, float* __restrict__ vf, float* __restrict__ decay,
                     float* __restrict__ beta) {
    __shared__ float sum_s[16];
    const int64_t t = t0 + blockIdx.x;
    const int unit = blockIdx.y;
    const int seq = token_seq[t];
    const int begin = cu_seqlens_q[seq];
    const int local = (int)t - begin;                                   // the token's place in its portion
    const bool has_past = seq_starts[seq] > 0;
    const int slot = state_slots[seq];
    const int qk = kv_heads * dim, vv = heads * vdim, channels = 2 * qk + vv;
    const int dp = (dim + 3) & ~3;
    const int tid = threadIdx.x;
    auto conv_silu = [&](int c) __attribute__((always_inline)) {
        float sum = 0.f;
        for (int j = 0; j < taps; ++j) {
            const int src = local - (taps - 1) + j;                     // < 0: before the portion
            float x = 0.f;
            if (src >= 0) x = to_float(proj[(int64_t)(begin + src) * stride + c]);
            else if (has_past) x = conv_state[((int64_t)slot * channels + c) * (taps - 1) + (taps - 1 + src)];
            sum += to_float(conv_w[(int64_t)c * taps + j]) * x;
        }
        return sum / (1.f + expf(-sum));
    };
    if (unit < 2 * kv_heads) {
        // a query or key head: its channels are unit * dim .. + dim of the row; the unit norm over the head
        constexpr int PER = (DELTA_MAX_DIM + DELTA_PREPARE_THREADS - 1) / DELTA_PREPARE_THREADS;
        float y[PER];
        float ss = 0.f;
#pragma unroll
        for (int i = 0; i < PER; ++i) {
            const int d = i * DELTA_PREPARE_THREADS + tid;
            y[i] = d < dim ? conv_silu(unit * dim + d) : 0.f;
            ss += y[i] * y[i];
        }
        ss = block_sum(ss, sum_s);
        const bool is_q = unit < kv_heads;
        float scale = 1.f / sqrtf(ss + 1e-6f);
        if (is_q) scale *= 1.f / sqrtf((float)dim);
        float* dst = (is_q ? qn + (t * kv_heads + unit) * dp : kn + (t * kv_heads + (unit - kv_heads)) * dp);
#pragma unroll
        for (int i = 0; i < PER; ++i) {
            const int d = i * DELTA_PREPARE_THREADS + tid;
            if (d < dp) dst[d] = y[i] * scale;                          // (zeros in the padding)
        }
        return;
    }
    const int h = unit - 2 * kv_heads;
    for (int d = tid; d < vdim; d += DELTA_PREPARE_THREADS) vf[t * vv + h * vdim + d] = conv_silu(2 * qk + h * vdim + d);
    const float rate = expf(a_log[h]);
    if (HEAD) {
        if (tid == 0) {
            decay[t * heads + h] = -rate * delta_softplus(delta_rate(rates, t, heads, heads + h) + dt_bias[h]);
            beta[t * heads + h] = 1.f / (1.f + expf(-delta_rate(rates, t, heads, h)));
        }
        return;
    }
    for (int d = tid; d < dp; d += DELTA_PREPARE_THREADS) {
        float a = 0.f;
        if (d < dim) {
            const float z = decay_in[t * (int64_t)(heads * dim) + h * dim + d] + dt_bias[h * dim + d];
            a = expf(-rate * delta_softplus(z));
        }
        decay[(t * heads + h) * dp + d] = a;
    }
    if (tid == 0) beta[t * heads + h] = 1.f / (1.f + expf(-to_float(proj[t * stride + channels + h])));
}

// One thread a (request, channel): the request's last taps - 1 inputs, from the portion where it is long enough,
// else from what was kept before (zeros at a request's start).
template <typename T>
__global__ void __launch_bounds__(256)
delta_keep_kernel(const T* __restrict__ proj, int64_t stride, float* __restrict__ conv_state,
                  const int32_t* __restrict__ cu_seqlens_q, const int32_t* __restrict__ seq_starts,
                  const int32_t* __restrict__ state_slots, int channels, int taps) {
    const int seq = blockIdx.y;
    const int c = blockIdx.x * blockDim.x + threadIdx.x;
    if (c >= channels) return;
    const int begin = cu_seqlens_q[seq], n = cu_seqlens_q[seq + 1] - begin;
    const bool has_past = seq_starts[seq] > 0;
    float* kept = conv_state + ((int64_t)state_slots[seq] * channels + c) * (taps - 1);
    float fresh[DELTA_MAX_TAPS];
    for (int i = 0; i < taps - 1; ++i) {
        const int src = n - (taps - 1) + i;
        fresh[i] = src >= 0 ? to_float(proj[(int64_t)(begin + src) * stride + c]) : has_past ? kept[taps - 1 + src] : 0.f;
    }
    for (int i = 0; i < taps - 1; ++i) kept[i] = fresh[i];
}

// The sum of x over the L = 8 or 16 neighbouring lanes that share a column of S: two exchanges inside the quads, then
// one between the two quads of every 8 lanes, which by then hold one value each, then one between the two eights.
template <int L>
__device__ __forceinline__ float delta_sum_lanes(float x) {
    x += __int_as_float(__builtin_amdgcn_update_dpp(0, __float_as_int(x), 0xB1, 0xF, 0xF, true));     // lanes 1 0 3 2
    x += __int_as_float(__builtin_amdgcn_update_dpp(0, __float_as_int(x), 0x4E, 0xF, 0xF, true));     // lanes 2 3 0 1
    x += __int_as_float(__builtin_amdgcn_update_dpp(0, __float_as_int(x), 0x141, 0xF, 0xF, true));    // lanes 7 .. 0 of each 8
    if (L == 16) x += __int_as_float(__builtin_amdgcn_update_dpp(0, __float_as_int(x), 0x140, 0xF, 0xF, true));   // 15 .. 0 of each 16
    return x;
}

// One workgroup of four waves per (request, head, 256 / L columns of S).  A column's DMAX rows (rows beyond D: zeros,
// with q, k and a staged as zeros) lie in L neighbouring lanes: lane r of them holds the rows 4 (r + L j) .. + 3 for
// j < DMAX / (4 L), so that the L lanes read consecutive floats of a staged row at a time.  Per token, in this order:
// S <- a S, u = beta (v - S^T k), S <- S + k u, o = S^T q; each of the two sums over the rows runs as four chains a
// lane and then over the L lanes, in an order that depends on D alone.  The tokens' q, k, a and beta go through LDS,
// a batch at a time in two buffers: the next batch is asked for before this one's sums and stored after them.
// HEAD: the decay is one number per token and head; S^T k is then summed over the state before the decay and multiplied
// by it, and the decay and the write are one fused operation an entry.
template <int DMAX, int L, bool HEAD>
__global__ void __launch_bounds__(DELTA_THREADS)
delta_scan_kernel(const float* __restrict__ qn, const float* __restrict__ kn, const float* __restrict__ vf,
                  const float* __restrict__ decay, const float* __restrict__ beta, float* __restrict__ o_raw,
                  float* __restrict__ state, const int32_t* __restrict__ cu_seqlens_q,
                  const int32_t* __restrict__ seq_starts, const int32_t* __restrict__ state_slots, int heads,
                  int kv_heads, int dim, int vdim) {
    constexpr int R4 = DMAX / (4 * L);                                  // float4s of rows a lane holds
    constexpr int COLS = DELTA_THREADS / L;                             // columns of S a workgroup holds
    constexpr int ROW4 = DMAX / 4;                                      // float4s of a staged row
    constexpr int ROWS = HEAD ? 2 : 3;                                  // q, k (and a, where it is a row)
    constexpr int STAGED4 = ROWS * DELTA_BATCH * ROW4;                  // staged a batch
    constexpr int NP = (STAGED4 + DELTA_THREADS - 1) / DELTA_THREADS;
    __shared__ float4 qka_s[2][ROWS][DELTA_BATCH][ROW4];
    __shared__ float beta_s[2][DELTA_BATCH], decay_s[2][DELTA_BATCH];
    const int seq = blockIdx.x, h = blockIdx.y, tid = threadIdx.x;
    const int r = tid % L;
    const int col = blockIdx.z * COLS + tid / L;
    const bool live = col < vdim;
    const int g = h / (heads / kv_heads);
    const int begin = cu_seqlens_q[seq], n = cu_seqlens_q[seq + 1] - begin;
    const int vv = heads * vdim;
    const int dp = (dim + 3) & ~3, dp4 = dp / 4;
    float* S_g = state + (((int64_t)state_slots[seq] * heads + h) * dim) * vdim + col;
    const bool has_past = seq_starts[seq] > 0;
    float S[4 * R4];
#pragma unroll
    for (int j = 0; j < R4; ++j)
#pragma unroll
        for (int e = 0; e < 4; ++e) {
            const int row = 4 * (r + L * j) + e;
            S[4 * j + e] = has_past && live && row < dim ? S_g[(int64_t)row * vdim] : 0.f;
        }

    // a batch's q, k, a (and beta) from global memory into registers, and from there into one of the two buffers
    float4 pre[NP];
    float pre_beta = 0.f, pre_decay = 0.f;
    auto ask = [&](int t0) __attribute__((always_inline)) {
        const int nb = min(DELTA_BATCH, n - t0);
#pragma unroll
        for (int i = 0; i < NP; ++i) {
            const int e = i * DELTA_THREADS + tid;
            const int which = e / (DELTA_BATCH * ROW4), b = (e / ROW4) % DELTA_BATCH, d4 = e % ROW4;
            float4 x = make_float4(0.f, 0.f, 0.f, 0.f);
            if (e < STAGED4 && b < nb && d4 < dp4) {
                const int64_t tok = begin + t0 + b;
                const float* row = which == 0 ? qn + (tok * kv_heads + g) * dp : which == 1 ? kn + (tok * kv_heads + g) * dp
                                                                                             : decay + (tok * heads + h) * dp;
                x = *reinterpret_cast<const float4*>(row + 4 * d4);
            }
            pre[i] = x;
        }
        pre_beta = tid < nb ? beta[(int64_t)(begin + t0 + tid) * heads + h] : 0.f;
        if (HEAD) pre_decay = tid < nb ? expf(decay[(int64_t)(begin + t0 + tid) * heads + h]) : 0.f;
    };
    auto put = [&](int buf) __attribute__((always_inline)) {
        float4* flat = &qka_s[buf][0][0][0];
#pragma unroll
        for (int i = 0; i < NP; ++i) {
            const int e = i * DELTA_THREADS + tid;
            if (e < STAGED4) flat[e] = pre[i];
        }
        if (tid < DELTA_BATCH) {
            beta_s[buf][tid] = pre_beta;
            if (HEAD) decay_s[buf][tid] = pre_decay;
        }
    };
    float v_next[DELTA_BATCH];
#pragma unroll
    for (int b = 0; b < DELTA_BATCH; ++b) v_next[b] = live && b < n ? vf[(int64_t)(begin + b) * vv + h * vdim + col] : 0.f;
    ask(0);
    put(0);
    __syncthreads();
    int buf = 0;
    for (int t0 = 0; t0 < n; t0 += DELTA_BATCH, buf ^= 1) {
        const int nb = min(DELTA_BATCH, n - t0);
        const bool more = t0 + DELTA_BATCH < n;
        if (more) ask(t0 + DELTA_BATCH);
        float v_now[DELTA_BATCH];
#pragma unroll
        for (int b = 0; b < DELTA_BATCH; ++b) {
            v_now[b] = v_next[b];
            const int tn = t0 + DELTA_BATCH + b;                        // the batch after: asked for now
            v_next[b] = live && tn < n ? vf[(int64_t)(begin + tn) * vv + h * vdim + col] : 0.f;
        }
        // a token's q, k, a and beta are read from LDS while the token before it is summed
        float4 a_c[R4], k_c[R4], q_c[R4];
        float beta_c, decay_c = 1.f;
        auto fetch = [&](int b, float4* a, float4* k, float4* q, float& be, float& de) __attribute__((always_inline)) {
#pragma unroll
            for (int j = 0; j < R4; ++j) {
                if (!HEAD) a[j] = qka_s[buf][ROWS - 1][b][r + L * j];
                k[j] = qka_s[buf][1][b][r + L * j];
                q[j] = qka_s[buf][0][b][r + L * j];
            }
            be = beta_s[buf][b];
            if (HEAD) de = decay_s[buf][b];
        };
        fetch(0, a_c, k_c, q_c, beta_c, decay_c);
#pragma unroll
        for (int b = 0; b < DELTA_BATCH; ++b) {
            if (b >= nb) break;
            float4 a_n[R4], k_n[R4], q_n[R4];
            float beta_n = 0.f, decay_n = 1.f;
            if (b + 1 < DELTA_BATCH) fetch(b + 1, a_n, k_n, q_n, beta_n, decay_n);      // (rows past the batch's last hold zeros)
            float d0 = 0.f, d1 = 0.f, d2 = 0.f, d3 = 0.f;
#pragma unroll
            for (int j = 0; j < R4; ++j) {
                const float4 k = k_c[j];
                if (!HEAD) {
                    const float4 a = a_c[j];
                    S[4 * j] *= a.x; S[4 * j + 1] *= a.y; S[4 * j + 2] *= a.z; S[4 * j + 3] *= a.w;
                }
                d0 += S[4 * j] * k.x; d1 += S[4 * j + 1] * k.y; d2 += S[4 * j + 2] * k.z; d3 += S[4 * j + 3] * k.w;
            }
            const float read = delta_sum_lanes<L>((d0 + d1) + (d2 + d3));
            const float u = beta_c * (v_now[b] - (HEAD ? decay_c * read : read));
            float o0 = 0.f, o1 = 0.f, o2 = 0.f, o3 = 0.f;
#pragma unroll
            for (int j = 0; j < R4; ++j) {
                const float4 k = k_c[j], q = q_c[j];
                if (HEAD) {
                    S[4 * j] = decay_c * S[4 * j] + k.x * u; S[4 * j + 1] = decay_c * S[4 * j + 1] + k.y * u;
                    S[4 * j + 2] = decay_c * S[4 * j + 2] + k.z * u; S[4 * j + 3] = decay_c * S[4 * j + 3] + k.w * u;
                } else {
                    S[4 * j] += k.x * u; S[4 * j + 1] += k.y * u; S[4 * j + 2] += k.z * u; S[4 * j + 3] += k.w * u;
                }
                o0 += S[4 * j] * q.x; o1 += S[4 * j + 1] * q.y; o2 += S[4 * j + 2] * q.z; o3 += S[4 * j + 3] * q.w;
            }
            const float o = delta_sum_lanes<L>((o0 + o1) + (o2 + o3));
            if (live && r == 0) o_raw[(int64_t)(begin + t0 + b) * vv + h * vdim + col] = o;
            if (b + 1 < DELTA_BATCH) {
#pragma unroll
                for (int j = 0; j < R4; ++j) {
                    if (!HEAD) a_c[j] = a_n[j];
                    k_c[j] = k_n[j], q_c[j] = q_n[j];
                }
                beta_c = beta_n;
                decay_c = decay_n;
            }
        }
        if (more) put(buf ^ 1);
        __syncthreads();                                                // the next batch is in; this one is done with
    }
    if (live) {
#pragma unroll
        for (int j = 0; j < R4; ++j)
#pragma unroll
            for (int e = 0; e < 4; ++e) {
                const int row = 4 * (r + L * j) + e;
                if (row < dim) S_g[(int64_t)row * vdim] = S[4 * j + e];
            }
    }
}

// SILU: the gate is silu(gate), else sigmoid(gate).
template <typename T, bool SILU>
__global__ void __launch_bounds__(NVA_WAVE)
delta_finish_kernel(const float* __restrict__ o_raw, const T* __restrict__ gate, int64_t gate_stride,
                    const float* __restrict__ norm_w, float eps, T* __restrict__ out, int64_t out_stride, int heads,
                    int vdim, int64_t t0) {
    const int64_t t = t0 + blockIdx.x;
    const int h = blockIdx.y, lane = threadIdx.x;
    const float* o = o_raw + (t * heads + h) * (int64_t)vdim;
    float ss = 0.f;
    for (int d = lane; d < vdim; d += NVA_WAVE) ss += o[d] * o[d];
    ss = wave_sum(ss);
    const float scale = 1.f / sqrtf(ss / (float)vdim + eps);
    for (int d = lane; d < vdim; d += NVA_WAVE) {
        const float z = to_float(gate[t * gate_stride + h * vdim + d]);
        const float gt = (SILU ? z : 1.f) / (1.f + expf(-z));
        out[t * out_stride + h * vdim + d] = from_float<T>(o[d] * scale * norm_w[d] * gt);
    }
}

// ---------------------------------------------------------------------------- single tokens, one decay per head
// One workgroup per (request, value head) of the requests that bring one token; token t of the step is request t's.
// Thread (r, c4) holds the columns 4 c4 .. + 3 of the rows r, r + RG, ... of S, CG = 512 / RG column groups (a power of
// two).  The two sums over the rows run inside a thread, then over the RG threads of a column in order.  keep: the
// workgroup also moves on the kept inputs of its channels (only where no other workgroup reads them: as many query/key
// heads as value heads).
template <typename T, int R>
__global__ void __launch_bounds__(DELTA_SINGLE_THREADS)
delta_single_kernel(const T* __restrict__ proj, int64_t stride, DeltaRates rates, const T* __restrict__ conv_w,
                    const float* __restrict__ dt_bias, const float* __restrict__ a_log, const float* __restrict__ norm_w,
                    float eps, float* __restrict__ s_state, float* __restrict__ conv_state,
                    const int32_t* __restrict__ seq_starts, const int32_t* __restrict__ state_slots, int heads, int kv_heads,
                    int dim, int vdim, int taps, int cg_log, int keep, T* __restrict__ out, int64_t out_stride) {
    extern __shared__ __attribute__((aligned(16))) float single_s[];
    __shared__ float scratch[16], sums_s[2];
    const int CG = 1 << cg_log, RG = DELTA_SINGLE_THREADS >> cg_log;
    const int vp = 4 * CG;                                              // columns, padded
    float* const row_s = single_s;                                      // [2 dim + vdim]: q, k, v
    float* const u_s = row_s + ((2 * dim + vdim + 3) & ~3);             // [vp]
    float* const red_s = u_s + vp;                                      // [RG][vp]
    const int64_t t = blockIdx.x;
    const int h = blockIdx.y, tid = threadIdx.x;
    const int g = h / (heads / kv_heads);
    const int qk = kv_heads * dim, vv = heads * vdim, channels = 2 * qk + vv;
    const int slot = state_slots[t];
    const bool has_past = seq_starts[t] > 0;
    const int c4 = tid & (CG - 1), r = tid >> cg_log;
    const bool live = 4 * c4 < vdim;
    float* S_g = s_state + ((int64_t)slot * heads + h) * dim * vdim + 4 * c4;
    delta_f32x4 S[R];
#pragma unroll
    for (int i = 0; i < R; ++i) {
        const int row = r + RG * i;
        S[i] = delta_f32x4{0.f, 0.f, 0.f, 0.f};
        if (has_past && live && row < dim) S[i] = *reinterpret_cast<const delta_f32x4*>(S_g + (int64_t)row * vdim);
    }
    const float gate_z = tid < vdim ? to_float(proj[t * stride + channels + h * vdim + tid]) : 0.f;
    const float a = expf(-expf(a_log[h]) * delta_softplus(delta_rate(rates, t, heads, heads + h) + dt_bias[h]));
    const float beta = 1.f / (1.f + expf(-delta_rate(rates, t, heads, h)));
    for (int i = tid; i < 2 * dim + vdim; i += DELTA_SINGLE_THREADS) {
        const int c = i < dim ? g * dim + i : i < 2 * dim ? qk + g * dim + (i - dim) : 2 * qk + h * vdim + (i - 2 * dim);
        float* kept = conv_state + ((int64_t)slot * channels + c) * (taps - 1);
        const float x = to_float(proj[t * stride + c]);
        float sum = 0.f;
        for (int j = 0; j < taps - 1; ++j) {
            const float old = has_past ? kept[j] : 0.f;
            sum += to_float(conv_w[(int64_t)c * taps + j]) * old;
            if (keep && j > 0) kept[j - 1] = old;
        }
        if (keep && taps > 1) kept[taps - 2] = x;
        sum += to_float(conv_w[(int64_t)c * taps + taps - 1]) * x;
        row_s[i] = sum / (1.f + expf(-sum));
    }
    __syncthreads();
    const int wave = tid / NVA_WAVE, lane = tid % NVA_WAVE;
    if (wave < 2) {
        float ss = 0.f;
        for (int d = lane; d < dim; d += NVA_WAVE) ss += row_s[wave * dim + d] * row_s[wave * dim + d];
        ss = wave_sum(ss);
        if (lane == 0) sums_s[wave] = ss;
    }
    __syncthreads();
    const float q_scale = (1.f / sqrtf(sums_s[0] + 1e-6f)) * (1.f / sqrtf((float)dim)), k_scale = 1.f / sqrtf(sums_s[1] + 1e-6f);
    float kr[R], qr[R];
    delta_f32x4 d = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int i = 0; i < R; ++i) {
        const int row = r + RG * i;
        kr[i] = row < dim ? row_s[dim + row] * k_scale : 0.f;
        qr[i] = row < dim ? row_s[row] * q_scale : 0.f;
#pragma unroll
        for (int e = 0; e < 4; ++e) d[e] += S[i][e] * kr[i];
    }
    *reinterpret_cast<delta_f32x4*>(&red_s[r * vp + 4 * c4]) = d;
    __syncthreads();
    if (tid < vp) {
        float read = 0.f;
        for (int i = 0; i < RG; ++i) read += red_s[i * vp + tid];
        u_s[tid] = tid < vdim ? beta * (row_s[2 * dim + tid] - a * read) : 0.f;
    }
    __syncthreads();
    const delta_f32x4 u = *reinterpret_cast<const delta_f32x4*>(&u_s[4 * c4]);
    delta_f32x4 o = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int i = 0; i < R; ++i) {
        const int row = r + RG * i;
#pragma unroll
        for (int e = 0; e < 4; ++e) {
            S[i][e] = a * S[i][e] + kr[i] * u[e];
            o[e] += S[i][e] * qr[i];
        }
        if (live && row < dim) *reinterpret_cast<delta_f32x4*>(S_g + (int64_t)row * vdim) = S[i];
    }
    *reinterpret_cast<delta_f32x4*>(&red_s[r * vp + 4 * c4]) = o;
    __syncthreads();
    float oc = 0.f;
    if (tid < vdim)
        for (int i = 0; i < RG; ++i) oc += red_s[i * vp + tid];
    const float ss = block_sum(oc * oc, scratch);
    const float scale = 1.f / sqrtf(ss / (float)vdim + eps);
    if (tid < vdim)
        out[t * out_stride + h * vdim + tid] = from_float<T>(oc * scale * norm_w[tid] * gate_z / (1.f + expf(-gate_z)));
}

// ---------------------------------------------------------------------------- portions in blocks, one decay per head
// units: int32 [n][4] = (request, the block's first token counted through the step, its tokens, unused); a portion's blocks
// side by side.  Scratch of block u and head h, each indexed by ub = u * heads + h: g_cum [ub][64], and the operands of the
// pass over the blocks as its lanes hold them, 64 x 4 floats side by side (one load a wave): w and q [ub][4 x 16 tokens]
// [KB x 16 channels], p [ub][4 x 16 tokens][4 x 16 tokens], k_t [ub][KB x 16 channels][4 x 16 tokens], all as left operands
// (row lane % 16, columns 4 (lane / 16) + j), u [ub][DV / 16][4 x 16 tokens] as results (rows 4 (lane / 16) + i, column
// lane % 16).  Tokens past a block's end are zeros in w, p, k_t and u.
template <typename T, int TAPS>
__global__ void __launch_bounds__(DELTA_PREPARE_THREADS)
delta_block_prepare_kernel(const T* __restrict__ proj, int64_t stride, DeltaRates rates, const T* __restrict__ conv_w,
                           const float* __restrict__ dt_bias, const float* __restrict__ a_log,
                           const float* __restrict__ conv_state, const int32_t* __restrict__ units,
                           const int32_t* __restrict__ cu_seqlens_q, const int32_t* __restrict__ seq_starts,
                           const int32_t* __restrict__ state_slots, int heads, int kv_heads, int dim, int vdim,
                           float* __restrict__ qn, float* __restrict__ kn, float* __restrict__ vf, float* __restrict__ decay,
                           float* __restrict__ beta) {
    constexpr int N = 16;                                               // tokens of a workgroup
    __shared__ float part_s[DELTA_PREPARE_THREADS / NVA_WAVE][N];
    const int32_t* un = units + 4 * (blockIdx.x / (DELTA_BLOCK / N));
    const int t0 = N * (blockIdx.x % (DELTA_BLOCK / N));
    const int seq = un[0], n = un[2] - t0;
    if (n <= 0) return;
    const int nt = min(n, N);
    const int64_t tok0 = un[1] + t0;
    const int begin = cu_seqlens_q[seq], local0 = (int)tok0 - begin;
    const bool has_past = seq_starts[seq] > 0;
    const int slot = state_slots[seq];
    const int qk = kv_heads * dim, vv = heads * vdim, channels = 2 * qk + vv;
    const int dp = (dim + 3) & ~3;
    const int unit = blockIdx.y, tid = threadIdx.x;
    auto conv_silu = [&](int c, float* y) __attribute__((always_inline)) {
        float w[TAPS], x[TAPS], in[N];
#pragma unroll
        for (int j = 0; j < TAPS; ++j) w[j] = to_float(conv_w[(int64_t)c * TAPS + j]);
#pragma unroll
        for (int i = 0; i < N; ++i) in[i] = to_float(proj[(tok0 + min(i, nt - 1)) * stride + c]);
#pragma unroll
        for (int j = 0; j < TAPS - 1; ++j) {
            const int src = local0 - (TAPS - 1) + j;                    // < 0: before the portion
            x[j] = 0.f;
            if (src >= 0) x[j] = to_float(proj[(int64_t)(begin + src) * stride + c]);
            else if (has_past) x[j] = conv_state[((int64_t)slot * channels + c) * (TAPS - 1) + (TAPS - 1 + src)];
        }
#pragma unroll
        for (int i = 0; i < N; ++i) {
            x[TAPS - 1] = in[i];
            float sum = 0.f;
#pragma unroll
            for (int j = 0; j < TAPS; ++j) sum += w[j] * x[j];
            y[i] = sum / (1.f + expf(-sum));
#pragma unroll
            for (int j = 0; j < TAPS - 1; ++j) x[j] = x[j + 1];
        }
    };
    if (unit < 2 * kv_heads) {
        constexpr int PER = (DELTA_MAX_DIM + DELTA_PREPARE_THREADS - 1) / DELTA_PREPARE_THREADS;
        float y[PER][N], ss[N];
#pragma unroll
        for (int i = 0; i < N; ++i) ss[i] = 0.f;
#pragma unroll
        for (int p = 0; p < PER; ++p) {
            const int d = p * DELTA_PREPARE_THREADS + tid;
#pragma unroll
            for (int i = 0; i < N; ++i) y[p][i] = 0.f;
            if (d < dim) conv_silu(unit * dim + d, y[p]);
#pragma unroll
            for (int i = 0; i < N; ++i) ss[i] += y[p][i] * y[p][i];
        }
#pragma unroll
        for (int i = 0; i < N; ++i) {
            const float s = wave_sum(ss[i]);
            if (tid % NVA_WAVE == 0) part_s[tid / NVA_WAVE][i] = s;
        }
        __syncthreads();
        const bool is_q = unit < kv_heads;
        float* dst = (is_q ? qn : kn) + (tok0 * kv_heads + (is_q ? unit : unit - kv_heads)) * dp;
#pragma unroll
        for (int i = 0; i < N; ++i) {
            if (i >= nt) break;
            float scale = 1.f / sqrtf(part_s[0][i] + part_s[1][i] + 1e-6f);
            if (is_q) scale *= 1.f / sqrtf((float)dim);
#pragma unroll
            for (int p = 0; p < PER; ++p) {
                const int d = p * DELTA_PREPARE_THREADS + tid;
                if (d < dp) dst[(int64_t)i * kv_heads * dp + d] = y[p][i] * scale;      // (zeros in the padding)
            }
        }
        return;
    }
    const int h = unit - 2 * kv_heads;
    for (int d = tid; d < vdim; d += DELTA_PREPARE_THREADS) {
        float y[N];
        conv_silu(2 * qk + h * vdim + d, y);
#pragma unroll
        for (int i = 0; i < N; ++i)
            if (i < nt) vf[(tok0 + i) * vv + h * vdim + d] = y[i];
    }
    if (tid < nt) {
        decay[(tok0 + tid) * heads + h] = -expf(a_log[h]) * delta_softplus(delta_rate(rates, tok0 + tid, heads, heads + h) + dt_bias[h]);
        beta[(tok0 + tid) * heads + h] = 1.f / (1.f + expf(-delta_rate(rates, tok0 + tid, heads, h)));
    }
}

// KB: steps of 16 key channels (dim <= 16 KB).  Products by v_mfma_f32_16x16x4_f32: lane l holds row (or column) l % 16 and,
// over the four instructions of a step of 16 channels, the channels 4 (l / 16) + j of both operands; results: row
// 4 (l / 16) + i, column l % 16.
template <int KB>
__global__ void __launch_bounds__(256)
delta_block_solve_kernel(const float* __restrict__ qn, const float* __restrict__ kn, const float* __restrict__ vf,
                         const float* __restrict__ decay, const float* __restrict__ beta, const int32_t* __restrict__ units,
                         int heads, int kv_heads, int dim, int vdim, float* __restrict__ g_cum, delta_f32x4* __restrict__ w_out,
                         delta_f32x4* __restrict__ q_out, delta_f32x4* __restrict__ u_out, delta_f32x4* __restrict__ p_out,
                         delta_f32x4* __restrict__ kt_out) {
    __shared__ __attribute__((aligned(16))) float tile_s[4][16][20];        // a wave's, to turn a result into a left operand
    __shared__ __attribute__((aligned(16))) float a_s[DELTA_BLOCK][DELTA_BLOCK + 4];
    __shared__ __attribute__((aligned(16))) float inv_s[4][16][20];
    __shared__ float g_s[DELTA_BLOCK], b_s[DELTA_BLOCK], bg_s[DELTA_BLOCK], eg_s[DELTA_BLOCK];
    const int h = blockIdx.x % heads;
    const int64_t ub = blockIdx.x;
    const int32_t* un = units + 4 * (blockIdx.x / heads);
    const int64_t first = un[1];
    const int n = un[2];
    const int kvh = h / (heads / kv_heads);
    const int dp = (dim + 3) & ~3, vv = heads * vdim;
    const int tid = threadIdx.x, wave = tid / NVA_WAVE, lane = tid % NVA_WAVE, col = lane & 15, g = lane >> 4;
    if (wave == 0) {
        float sum = lane < n ? decay[(first + lane) * heads + h] : 0.f;
#pragma unroll
        for (int off = 1; off < NVA_WAVE; off <<= 1) {
            const float up = __shfl_up(sum, off, NVA_WAVE);
            if (lane >= off) sum += up;
        }
        const float be = lane < n ? beta[(first + lane) * heads + h] : 0.f;
        g_s[lane] = sum;
        b_s[lane] = be;
        bg_s[lane] = be * expf(sum);
        eg_s[lane] = expf(__shfl(sum, NVA_WAVE - 1, NVA_WAVE) - sum);
        g_cum[ub * DELTA_BLOCK + lane] = sum;
    }
    __syncthreads();
    // a wave's 16 x 16 result (rows 4 g + i, column col) as a left operand (row col, columns 4 g + j)
    auto turned = [&](const delta_f32x4& v) __attribute__((always_inline)) {
#pragma unroll
        for (int i = 0; i < 4; ++i) tile_s[wave][4 * g + i][col] = v[i];
        return *reinterpret_cast<const delta_f32x4*>(&tile_s[wave][col][4 * g]);
    };
    // the ten blocks of 16 x 16 on and below the diagonal, of k k^T and of q k^T
    for (int task = wave; task < 20; task += 4) {
        const int pair = task >> 1;
        const bool of_q = task & 1;
        const int bi = pair < 1 ? 0 : pair < 3 ? 1 : pair < 6 ? 2 : 3, bj = pair - bi * (bi + 1) / 2;
        const float* ar = (of_q ? qn : kn) + ((first + min(16 * bi + col, n - 1)) * kv_heads + kvh) * dp + 4 * g;
        const float* br = kn + ((first + min(16 * bj + col, n - 1)) * kv_heads + kvh) * dp + 4 * g;
        delta_f32x4 fa[KB], fb[KB];
#pragma unroll
        for (int s = 0; s < KB; ++s) {
            fa[s] = fb[s] = delta_f32x4{0.f, 0.f, 0.f, 0.f};
            if (16 * s + 4 * g < dp) {
                fa[s] = *reinterpret_cast<const delta_f32x4*>(ar + 16 * s);
                fb[s] = *reinterpret_cast<const delta_f32x4*>(br + 16 * s);
            }
        }
        delta_f32x4 acc = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int s = 0; s < KB; ++s)
#pragma unroll
            for (int j = 0; j < 4; ++j) acc = __builtin_amdgcn_mfma_f32_16x16x4f32(fa[s][j], fb[s][j], acc, 0, 0, 0);
        delta_f32x4 v;
#pragma unroll
        for (int i = 0; i < 4; ++i) {
            const int r = 16 * bi + 4 * g + i, c = 16 * bj + col;
            const bool seen = r < n && (of_q ? c <= r : c < r);
            v[i] = seen ? expf(g_s[r] - g_s[c]) * acc[i] : 0.f;
            if (!of_q) a_s[r][c] = b_s[r] * v[i];
        }
        if (of_q) {
            p_out[((ub * 4 + bi) * 4 + bj) * NVA_WAVE + lane] = turned(v);
            if (bj == 0) {
#pragma unroll
                for (int s = 0; s < KB; ++s) q_out[((ub * 4 + bi) * KB + s) * NVA_WAVE + lane] = fa[s];
            }
        }
    }
    __syncthreads();
    // the inverses of the four diagonal blocks of I + A: wave w's of block w, a lane a column, row by row
    {
        float x[16];
        const int b0 = 16 * wave;
#pragma unroll
        for (int i = 0; i < 16; ++i) {
            float s[4] = {i == col ? 1.f : 0.f, 0.f, 0.f, 0.f};
#pragma unroll
            for (int j = 0; j < i; j += 4) {
                const delta_f32x4 av = *reinterpret_cast<const delta_f32x4*>(&a_s[b0 + i][b0 + j]);
#pragma unroll
                for (int e = 0; e < 4; ++e)
                    if (j + e < i) s[e] -= av[e] * x[j + e];
            }
            x[i] = (s[0] + s[1]) + (s[2] + s[3]);
        }
        if (g == 0) {
#pragma unroll
            for (int i = 0; i < 16; ++i) inv_s[wave][i][col] = x[i];
        }
    }
    __syncthreads();
    // Block rows of A (negated) and the inverses as left operands: row lane % 16, columns 4 (lane / 16) + j.  A result of a
    // product (rows 4 (lane / 16) + i) is the right operand of the next as it stands.
    delta_f32x4 af[6], inv[4];
#pragma unroll
    for (int bi = 0; bi < 4; ++bi) {
        inv[bi] = *reinterpret_cast<const delta_f32x4*>(&inv_s[bi][col][4 * g]);
#pragma unroll
        for (int bj = 0; bj < bi; ++bj) {
            const delta_f32x4 v = *reinterpret_cast<const delta_f32x4*>(&a_s[16 * bi + col][16 * bj + 4 * g]);
            af[bi * (bi - 1) / 2 + bj] = delta_f32x4{-v[0], -v[1], -v[2], -v[3]};
        }
    }
    // forward substitution by blocks of 16 rows: a wave 16 columns at a time, of beta v (the first DV) or of beta exp(G) k
    // (columns past a size repeat the last one: the pass over the blocks meets them with zeros, or writes nothing of them)
    const int v_blocks = (vdim + 15) / 16, blocks = v_blocks + KB;
    for (int cb = wave; cb < blocks; cb += 4) {
        const bool of_v = cb < v_blocks;
        const int d = 16 * (of_v ? cb : cb - v_blocks) + col, width = of_v ? vdim : dp;
        const float* src = of_v ? vf + first * vv + h * vdim : kn + (first * kv_heads + kvh) * dp;
        const int64_t step = of_v ? vv : (int64_t)kv_heads * dp;
        const float* scale = of_v ? b_s : bg_s;                         // (zero past the block's end)
        delta_f32x4 x[4];
#pragma unroll
        for (int bi = 0; bi < 4; ++bi)
#pragma unroll
            for (int i = 0; i < 4; ++i) x[bi][i] = src[min(16 * bi + 4 * g + i, n - 1) * step + min(d, width - 1)];
        if (!of_v) {
#pragma unroll
            for (int bi = 0; bi < 4; ++bi) {
                delta_f32x4 v;
#pragma unroll
                for (int i = 0; i < 4; ++i) {
                    const int t = 16 * bi + 4 * g + i;
                    v[i] = t < n ? x[bi][i] * eg_s[t] : 0.f;
                }
                kt_out[((ub * KB + cb - v_blocks) * 4 + bi) * NVA_WAVE + lane] = v;
            }
        }
#pragma unroll
        for (int bi = 0; bi < 4; ++bi) {
            delta_f32x4 r;
#pragma unroll
            for (int i = 0; i < 4; ++i) r[i] = x[bi][i] * scale[16 * bi + 4 * g + i];
#pragma unroll
            for (int bj = 0; bj < bi; ++bj)
#pragma unroll
                for (int j = 0; j < 4; ++j) r = __builtin_amdgcn_mfma_f32_16x16x4f32(af[bi * (bi - 1) / 2 + bj][j], x[bj][j], r, 0, 0, 0);
            delta_f32x4 y = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
            for (int j = 0; j < 4; ++j) y = __builtin_amdgcn_mfma_f32_16x16x4f32(inv[bi][j], r[j], y, 0, 0, 0);
            x[bi] = y;
        }
#pragma unroll
        for (int bi = 0; bi < 4; ++bi) {
            if (of_v) u_out[((ub * v_blocks + cb) * 4 + bi) * NVA_WAVE + lane] = x[bi];
            else w_out[((ub * 4 + bi) * KB + cb - v_blocks) * NVA_WAVE + lane] = turned(x[bi]);
        }
    }
}

// The workgroup's barrier, after this wave's own LDS traffic is done (loads on their way into registers are not waited for).
__device__ __forceinline__ void delta_barrier() { asm volatile("s_waitcnt lgkmcnt(0)\n\ts_barrier" ::: "memory"); }

// chains: int32 [n][4] = (a portion's first block, its blocks, its request, unused).  One workgroup of four waves per (head,
// portion, 16 columns of S), heads fastest, so that the workgroups of a head meet in one die's L2.  The state's columns lie
// in accumulators (wave w: the blocks w, w + 4, ... of 16 rows) and, transposed, in LDS for the products that read them.
template <int KB>
__global__ void __launch_bounds__(256) __attribute__((amdgpu_waves_per_eu(1, 1)))
delta_block_scan_kernel(const float* __restrict__ g_cum, const delta_f32x4* __restrict__ w_in, const delta_f32x4* __restrict__ q_in,
                        const delta_f32x4* __restrict__ u_in, const delta_f32x4* __restrict__ p_in,
                        const delta_f32x4* __restrict__ kt_in, float* __restrict__ o_raw, float* __restrict__ state, const int32_t* __restrict__ units,
                        const int32_t* __restrict__ chains, int num_chains, const int32_t* __restrict__ seq_starts,
                        const int32_t* __restrict__ state_slots, int heads, int dim, int vdim) {
    constexpr int NB = (KB + 3) / 4;
    __shared__ __attribute__((aligned(16))) float s_s[16][16 * KB + 4];     // [column][row]
    __shared__ __attribute__((aligned(16))) float u_s[16][DELTA_BLOCK + 4]; // [column][token]
    const int h = blockIdx.x % heads, rest = blockIdx.x / heads;
    const int32_t* ch = chains + 4 * (rest % num_chains);
    const int unit0 = ch[0], blocks = ch[1], seq = ch[2];
    const int tid = threadIdx.x, wave = __builtin_amdgcn_readfirstlane(tid / NVA_WAVE), lane = tid % NVA_WAVE, col = lane & 15, g = lane >> 4;
    const int column = 16 * (rest / num_chains) + col;
    const bool live = column < vdim;
    const int vv = heads * vdim, v_blocks = (vdim + 15) / 16;
    float* S_g = state + ((int64_t)state_slots[seq] * heads + h) * dim * vdim + column;
    const bool has_past = seq_starts[seq] > 0;
    delta_f32x4 S[NB];
#pragma unroll
    for (int b = 0; b < NB; ++b) {
        const int kb = wave + 4 * b;
#pragma unroll
        for (int i = 0; i < 4; ++i) {
            const int row = 16 * kb + 4 * g + i;
            S[b][i] = has_past && live && row < dim ? S_g[(int64_t)row * vdim] : 0.f;
        }
        if (kb < KB) *reinterpret_cast<delta_f32x4*>(&s_s[col][16 * kb + 4 * g]) = S[b];
    }
    // A block's operands, asked for while the block before it is at work.
    struct Operands {
        delta_f32x4 wf[KB], qf[KB], pf[4], kt[NB][4], gi, u;
        float g_end;
        int first, n;
    };
    // (Unconditional, the last block's once more behind the end: a load that may or may not be on its way makes every wait
    // before its use wait for all of them.)
    auto ask = [&](int blk, Operands& o) __attribute__((always_inline)) {
        blk = min(blk, blocks - 1);
        const int32_t* un = units + 4 * (unit0 + blk);
        const int64_t ub = (int64_t)(unit0 + blk) * heads + h;
        o.first = un[1], o.n = un[2];
        const delta_f32x4* wr = w_in + (ub * 4 + wave) * KB * NVA_WAVE + lane;
        const delta_f32x4* qr = q_in + (ub * 4 + wave) * KB * NVA_WAVE + lane;
        const delta_f32x4* pr = p_in + (ub * 4 + wave) * 4 * NVA_WAVE + lane;
        const float* gr = g_cum + ub * DELTA_BLOCK;
#pragma unroll
        for (int s = 0; s < KB; ++s) {
            o.wf[s] = wr[s * NVA_WAVE];
            o.qf[s] = qr[s * NVA_WAVE];
        }
        o.u = u_in[((ub * v_blocks + rest / num_chains) * 4 + wave) * NVA_WAVE + lane];
#pragma unroll
        for (int s = 0; s < 4; ++s) o.pf[s] = pr[(s <= wave ? s : 0) * NVA_WAVE];
#pragma unroll
        for (int b = 0; b < NB; ++b)
#pragma unroll
            for (int s = 0; s < 4; ++s) o.kt[b][s] = kt_in[((ub * KB + min(wave + 4 * b, KB - 1)) * 4 + s) * NVA_WAVE + lane];
        o.gi = *reinterpret_cast<const delta_f32x4*>(gr + 16 * wave + 4 * g);
        o.g_end = gr[DELTA_BLOCK - 1];
    };
    auto run = [&](const Operands& o) __attribute__((always_inline)) {
        // W S and Q S of this wave's 16 tokens
        delta_f32x4 x = {0.f, 0.f, 0.f, 0.f}, y = {0.f, 0.f, 0.f, 0.f}, sv[2];
        sv[0] = *reinterpret_cast<const delta_f32x4*>(&s_s[col][4 * g]);
#pragma unroll
        for (int s = 0; s < KB; ++s) {
            // (a step's operand is read from LDS while the step before it multiplies)
            if (s + 1 < KB) sv[(s + 1) & 1] = *reinterpret_cast<const delta_f32x4*>(&s_s[col][16 * (s + 1) + 4 * g]);
            __builtin_amdgcn_sched_barrier(0);
#pragma unroll
            for (int j = 0; j < 4; ++j) {
                x = __builtin_amdgcn_mfma_f32_16x16x4f32(o.wf[s][j], sv[s & 1][j], x, 0, 0, 0);
                y = __builtin_amdgcn_mfma_f32_16x16x4f32(o.qf[s][j], sv[s & 1][j], y, 0, 0, 0);
            }
            __builtin_amdgcn_sched_barrier(0);
        }
        delta_f32x4 u;
#pragma unroll
        for (int i = 0; i < 4; ++i) u[i] = o.u[i] - x[i], y[i] *= expf(o.gi[i]);
        *reinterpret_cast<delta_f32x4*>(&u_s[col][16 * wave + 4 * g]) = u;
        delta_barrier();                                                // the block's writes are in; the state is read
        const float e_end = expf(o.g_end);
#pragma unroll
        for (int b = 0; b < NB; ++b)
#pragma unroll
            for (int i = 0; i < 4; ++i) S[b][i] *= e_end;
        delta_f32x4 uv[4];
#pragma unroll
        for (int s = 0; s < 4; ++s) uv[s] = *reinterpret_cast<const delta_f32x4*>(&u_s[col][16 * s + 4 * g]);
        __builtin_amdgcn_sched_barrier(0);
#pragma unroll
        for (int s = 0; s < 4; ++s)
#pragma unroll
            for (int j = 0; j < 4; ++j)
#pragma unroll
                for (int b = 0; b < NB; ++b) S[b] = __builtin_amdgcn_mfma_f32_16x16x4f32(o.kt[b][s][j], uv[s][j], S[b], 0, 0, 0);
#pragma unroll
        for (int s = 0; s < 4; ++s)
            if (s <= wave)
#pragma unroll
                for (int j = 0; j < 4; ++j) y = __builtin_amdgcn_mfma_f32_16x16x4f32(o.pf[s][j], uv[s][j], y, 0, 0, 0);
        // (the state's rows past the head's size stay zero: the products that read them meet anything there)
#pragma unroll
        for (int b = 0; b < NB; ++b)
            if (wave + 4 * b < KB) {
                delta_f32x4 v = S[b];
#pragma unroll
                for (int i = 0; i < 4; ++i) v[i] = 16 * (wave + 4 * b) + 4 * g + i < dim ? v[i] : 0.f;
                *reinterpret_cast<delta_f32x4*>(&s_s[col][16 * (wave + 4 * b) + 4 * g]) = v;
            }
#pragma unroll
        for (int i = 0; i < 4; ++i) {
            const int row = 16 * wave + 4 * g + i;
            if (live && row < o.n) o_raw[(int64_t)(o.first + row) * vv + h * vdim + column] = y[i];
        }
        delta_barrier();                                                // the state is in; the block's writes are read
    };
    Operands even, odd;
    ask(0, even);
    delta_barrier();
    for (int blk = 0; blk < blocks; blk += 2) {
        ask(blk + 1, odd);
        run(even);
        if (blk + 1 >= blocks) break;
        ask(blk + 2, even);
        run(odd);
    }
    if (!live) return;
#pragma unroll
    for (int b = 0; b < NB; ++b)
#pragma unroll
        for (int i = 0; i < 4; ++i) {
            const int row = 16 * (wave + 4 * b) + 4 * g + i;
            if (row < dim) S_g[(int64_t)row * vdim] = S[b][i];
        }
}

// What both forms of the rule check.
static int check_delta(const char* what, const void* proj, int64_t stride, int64_t need, float* scratch, void* out,
                       int64_t out_stride, float* s_state, float* conv_state, const int32_t* token_seq,
                       const int32_t* cu_seqlens_q, const int32_t* seq_starts, const int32_t* state_slots, int64_t seqs,
                       int64_t tokens, int heads, int kv_heads, int dim, int vdim, int taps, const void* conv_w,
                       const float* dt_bias, const float* a_log, const float* norm_w) {
    if (tokens < 0 || tokens > 0x7fffffff || seqs <= 0 || seqs > 65535)
        return nva_fail("%s: bad counts tokens=%lld requests=%lld", what, (long long)tokens, (long long)seqs);
    if (heads <= 0 || kv_heads <= 0 || heads % kv_heads || heads > 65535 || dim <= 0 || vdim <= 0)
        return nva_fail("%s: bad sizes heads=%d kv_heads=%d dim=%d vdim=%d", what, heads, kv_heads, dim, vdim);
    if (dim > DELTA_MAX_DIM) return nva_fail("%s: a head of %d key channels (up to %d)", what, dim, DELTA_MAX_DIM);
    if (taps < 1 || taps > DELTA_MAX_TAPS) return nva_fail("%s: %d taps (1 to %d)", what, taps, DELTA_MAX_TAPS);
    if (!proj || stride < need || !scratch || !out || out_stride < heads * (int64_t)vdim || !s_state || (taps > 1 && !conv_state) ||
        !token_seq || !cu_seqlens_q || !seq_starts || !state_slots || !conv_w || !dt_bias || !a_log || !norm_w)
        return nva_fail("%s: a tensor is missing or too narrow", what);
    if (2 * (int64_t)kv_heads + heads > 65535) return nva_fail("%s: %d heads", what, heads);
    if ((uintptr_t)scratch % 16) return nva_fail("%s: the scratch memory must be 16-byte aligned", what);
    return 0;
}

// The request's recurrence token by token, 16 lanes a column where a head has rows for them (twice the waves, half the sums
// a lane), else 8.  The requests are the `seqs` from the pointers on.
template <bool HEAD>
static void launch_delta_scan(const float* qn, const float* kn, const float* vf, const float* decay, const float* beta, float* o_raw,
                              float* s_state, const int32_t* cu_seqlens_q, const int32_t* seq_starts, const int32_t* state_slots,
                              int64_t seqs, int heads, int kv_heads, int dim, int vdim, hipStream_t stream) {
#define DELTA_SCAN(DM, LL)                                                                                                \
    hipLaunchKernelGGL((delta_scan_kernel<DM, LL, HEAD>), dim3((unsigned)seqs, (unsigned)heads, (vdim + DELTA_THREADS / LL - 1) / (DELTA_THREADS / LL)), \
                       dim3(DELTA_THREADS), 0, stream, qn, kn, vf, decay, beta, o_raw, s_state, cu_seqlens_q, seq_starts,   \
                       state_slots, heads, kv_heads, dim, vdim)
    if (dim <= 32) DELTA_SCAN(32, 8); else if (dim <= 64) DELTA_SCAN(64, 16); else if (dim <= 128) DELTA_SCAN(128, 16); else DELTA_SCAN(256, 16);
#undef DELTA_SCAN
}

static void launch_delta_keep(const void* proj, int64_t stride, float* conv_state, const int32_t* cu_seqlens_q,
                              const int32_t* seq_starts, const int32_t* state_slots, int64_t seqs, int channels, int taps,
                              hipStream_t stream) {
    if (taps > 1 && seqs > 0)
        hipLaunchKernelGGL(delta_keep_kernel<elem_t>, dim3((channels + 255) / 256, (unsigned)seqs), dim3(256), 0, stream,
                           (const elem_t*)proj, stride, conv_state, cu_seqlens_q, seq_starts, state_slots, channels, taps);
}

// proj: elements [tokens, 2 G D + H DV + H], rows `stride` apart.  decay_in: float [tokens, H D].  gate_in: elements
// [tokens, H DV], rows gate_stride apart.  conv_w: elements [2 G D + H DV, taps].  dt_bias float [H D], a_log float [H],
// norm_w float [DV].  conv_state float [slots, 2 G D + H DV, taps - 1], s_state float [slots, H, D, DV]: a request's
// rows by state_slots, taken as zero where seq_starts is 0.  scratch: float [tokens * ((2 G + H) DP + 2 H DV + H)], DP = D rounded up to 4, 16-byte aligned.
// The step's requests by cu_seqlens_q [seqs + 1]; token_seq [tokens].  out: elements [tokens, H DV].
NVA_EXPORT int NVA_NAME(nva_channel_delta)(const void* proj, int64_t stride, const float* decay_in, const void* gate_in,
                                           int64_t gate_stride, float* scratch, void* out, int64_t out_stride,
                                           float* s_state, float* conv_state, const int32_t* token_seq,
                                           const int32_t* cu_seqlens_q, const int32_t* seq_starts,
                                           const int32_t* state_slots, int64_t seqs, int64_t tokens, int heads,
                                           int kv_heads, int dim, int vdim, int taps, const void* conv_w,
                                           const float* dt_bias, const float* a_log, const float* norm_w, float eps,
                                           hipStream_t stream) {
    if (tokens == 0) return 0;
    const int qk = kv_heads * dim, vv = heads * vdim, channels = 2 * qk + vv;
    const int bad = check_delta("channel_delta", proj, stride, channels + (int64_t)heads, scratch, out, out_stride, s_state, conv_state,
                                token_seq, cu_seqlens_q, seq_starts, state_slots, seqs, tokens, heads, kv_heads, dim, vdim, taps, conv_w,
                                dt_bias, a_log, norm_w);
    if (bad) return bad;
    if (!decay_in || !gate_in || gate_stride < vv) return nva_fail("channel_delta: a tensor is missing or too narrow");
    // scratch: q, k and the decays in rows of dim rounded up to 4 floats, then v, the read-outs and beta
    const int dp = (dim + 3) & ~3;
    float* qn = scratch;
    float* kn = qn + tokens * kv_heads * dp;
    float* decay = kn + tokens * kv_heads * dp;
    float* vf = decay + tokens * (int64_t)heads * dp;
    float* o_raw = vf + tokens * vv;
    float* beta = o_raw + tokens * vv;
    hipLaunchKernelGGL((delta_prepare_kernel<elem_t, false>), dim3((unsigned)tokens, (unsigned)(2 * kv_heads + heads)),
                       dim3(DELTA_PREPARE_THREADS), 0, stream, (const elem_t*)proj, stride, decay_in, DeltaRates{nullptr, 0, 0},
                       (int64_t)0, (const elem_t*)conv_w, dt_bias, a_log, conv_state, token_seq, cu_seqlens_q, seq_starts, state_slots,
                       heads, kv_heads, dim, vdim, taps, qn, kn, vf, decay, beta);
    launch_delta_keep(proj, stride, conv_state, cu_seqlens_q, seq_starts, state_slots, seqs, channels, taps, stream);
    launch_delta_scan<false>(qn, kn, vf, decay, beta, o_raw, s_state, cu_seqlens_q, seq_starts, state_slots, seqs, heads, kv_heads, dim,
                             vdim, stream);
    hipLaunchKernelGGL((delta_finish_kernel<elem_t, false>), dim3((unsigned)tokens, (unsigned)heads), dim3(NVA_WAVE), 0, stream, o_raw,
                       (const elem_t*)gate_in, gate_stride, norm_w, eps, (elem_t*)out, out_stride, heads, vdim, (int64_t)0);
    return nva_check_launch("channel_delta");
}

// The form for single tokens: how a head's columns are shared out, or -1 where it does not take the sizes.
static int delta_single_groups(int dim, int vdim) {
    if (vdim % 4 || vdim > DELTA_SINGLE_THREADS || dim > DELTA_MAX_DIM) return -1;
    int cg = 0;
    while ((4 << cg) < vdim) ++cg;
    const int rg = DELTA_SINGLE_THREADS >> cg;
    return rg >= 1 && (dim + rg - 1) / rg <= 16 ? cg : -1;
}

// Steps of 16 key channels that the blocks' kernels are built for.
static int delta_steps(int dim) { return dim <= 32 ? 2 : dim <= 64 ? 4 : dim <= 128 ? 8 : 16; }

// Floats that nva_head_delta's block_scratch holds for n blocks of portions.
NVA_EXPORT int64_t NVA_NAME(nva_head_delta_block_floats)(int64_t n, int heads, int dim, int vdim) {
    return n * heads * DELTA_BLOCK * (3 * 16 * (int64_t)delta_steps(dim) + (vdim + 15) / 16 * 16 + DELTA_BLOCK + 1);
}

// One decay per head.  proj: elements [tokens, 2 G D + 2 H DV] = [q | k | v | gate], rows `stride` apart.  rates: float
// [rate_splits][tokens, 2 H] = [b | a], the splits rate_stride apart and added up here.  dt_bias and a_log float [H].  scratch:
// float [tokens * (2 G DP + 2 H DV + 2 H)], 16-byte aligned.  The first `singles` requests bring one token each, which
// single_kernel (1 or 0) may take in a kernel of its own.  units [n_units][4] and chains [n_chains][4] (see the kernels) with
// block_scratch cover the other requests, which then run in blocks; n_units 0: token by token.  Everything else as for
// nva_channel_delta.
NVA_EXPORT int NVA_NAME(nva_head_delta)(const void* proj, int64_t stride, const float* rates, int rate_splits, int64_t rate_stride,
                                        float* scratch, void* out, int64_t out_stride, float* s_state, float* conv_state,
                                        const int32_t* token_seq, const int32_t* cu_seqlens_q, const int32_t* seq_starts,
                                        const int32_t* state_slots, int64_t seqs, int64_t tokens, int64_t singles,
                                        int single_kernel, int heads, int kv_heads, int dim, int vdim, int taps,
                                        const void* conv_w, const float* dt_bias, const float* a_log, const float* norm_w,
                                        float eps, const int32_t* units, int64_t n_units, const int32_t* chains,
                                        int64_t n_chains, float* block_scratch, hipStream_t stream) {
    if (tokens == 0) return 0;
    const int qk = kv_heads * dim, vv = heads * vdim, channels = 2 * qk + vv;
    const int bad = check_delta("head_delta", proj, stride, channels + (int64_t)vv, scratch, out, out_stride, s_state, conv_state, token_seq,
                                cu_seqlens_q, seq_starts, state_slots, seqs, tokens, heads, kv_heads, dim, vdim, taps, conv_w, dt_bias,
                                a_log, norm_w);
    if (bad) return bad;
    if (!rates || rate_splits <= 0 || (rate_splits > 1 && rate_stride < tokens * 2 * heads) || singles < 0 || singles > seqs)
        return nva_fail("head_delta: bad rates (%d splits) or %lld single tokens of %lld requests", rate_splits, (long long)singles, (long long)seqs);
    if (n_units && (!units || !chains || n_chains <= 0 || !block_scratch || (uintptr_t)block_scratch % 16 || n_units < n_chains ||
                    n_units * heads * (DELTA_BLOCK / 16) > 0x7fffffff || n_chains * heads * (int64_t)((vdim + 15) / 16) > 0x7fffffff))
        return nva_fail("head_delta: bad blocks (%lld in %lld portions)", (long long)n_units, (long long)n_chains);
    const DeltaRates rt{rates, rate_splits, rate_stride};
    const elem_t* pr = (const elem_t*)proj;
    const elem_t* cw = (const elem_t*)conv_w;
    const int cg = single_kernel && singles ? delta_single_groups(dim, vdim) : -1;
    if (cg >= 0) {
        const int rg = DELTA_SINGLE_THREADS >> cg, rows = (dim + rg - 1) / rg, keep = heads == kv_heads ? 1 : 0;
        const size_t lds = (size_t)(((2 * dim + vdim + 3) & ~3) + (4 << cg) + rg * (4 << cg)) * sizeof(float);
#define DELTA_SINGLE(RR)                                                                                                  \
        hipLaunchKernelGGL((delta_single_kernel<elem_t, RR>), dim3((unsigned)singles, (unsigned)heads), dim3(DELTA_SINGLE_THREADS),  \
                           lds, stream, pr, stride, rt, cw, dt_bias, a_log, norm_w, eps, s_state, conv_state, seq_starts, state_slots, \
                           heads, kv_heads, dim, vdim, taps, cg, keep, (elem_t*)out, out_stride)
        if (rows <= 1) DELTA_SINGLE(1); else if (rows <= 2) DELTA_SINGLE(2); else if (rows <= 4) DELTA_SINGLE(4);
        else if (rows <= 8) DELTA_SINGLE(8); else DELTA_SINGLE(16);
#undef DELTA_SINGLE
        if (!keep) launch_delta_keep(proj, stride, conv_state, cu_seqlens_q, seq_starts, state_slots, singles, channels, taps, stream);
    }
    // what is left: requests from first_seq on, whose tokens start at first (a single token a request before them)
    const int64_t first = cg >= 0 ? singles : 0, left = tokens - first;
    if (left <= 0) return nva_check_launch("head_delta");
    const int dp = (dim + 3) & ~3;
    float* qn = scratch;
    float* kn = qn + tokens * kv_heads * dp;
    float* vf = kn + tokens * kv_heads * dp;
    float* o_raw = vf + tokens * vv;
    float* beta = o_raw + tokens * vv;
    float* decay = beta + tokens * heads;
    const int64_t blocked_from = n_units ? singles : seqs;              // requests that run in blocks
    const int64_t plain_tokens = n_units ? singles - first : left;      // tokens of [first, ...) that run one by one
    const unsigned heads_y = (unsigned)(2 * kv_heads + heads);
    auto prepare = [&](int64_t t0, int64_t count) {
        if (count > 0)
            hipLaunchKernelGGL((delta_prepare_kernel<elem_t, true>), dim3((unsigned)count, heads_y), dim3(DELTA_PREPARE_THREADS), 0, stream,
                               pr, stride, (const float*)nullptr, rt, t0, cw, dt_bias, a_log, conv_state, token_seq, cu_seqlens_q,
                               seq_starts, state_slots, heads, kv_heads, dim, vdim, taps, qn, kn, vf, decay, beta);
    };
    if (n_units && taps <= 4) {
        prepare(first, plain_tokens);
        const dim3 grid((unsigned)(n_units * (DELTA_BLOCK / 16)), heads_y);
#define DELTA_BLOCK_PREPARE(TT)                                                                                           \
        hipLaunchKernelGGL((delta_block_prepare_kernel<elem_t, TT>), grid, dim3(DELTA_PREPARE_THREADS), 0, stream, pr, stride, rt, cw, \
                           dt_bias, a_log, conv_state, units, cu_seqlens_q, seq_starts, state_slots, heads, kv_heads, dim, vdim, qn, kn, \
                           vf, decay, beta)
        if (taps == 1) DELTA_BLOCK_PREPARE(1); else if (taps == 2) DELTA_BLOCK_PREPARE(2);
        else if (taps == 3) DELTA_BLOCK_PREPARE(3); else DELTA_BLOCK_PREPARE(4);
#undef DELTA_BLOCK_PREPARE
    } else {
        prepare(first, left);
    }
    launch_delta_keep(proj, stride, conv_state, cu_seqlens_q + first, seq_starts + first, state_slots + first, seqs - first, channels,
                      taps, stream);
    if (blocked_from > first)
        launch_delta_scan<true>(qn, kn, vf, decay, beta, o_raw, s_state, cu_seqlens_q + first, seq_starts + first, state_slots + first,
                                blocked_from - first, heads, kv_heads, dim, vdim, stream);
    if (n_units) {
        const int64_t rows = n_units * heads * DELTA_BLOCK;
        const unsigned slices = (unsigned)((vdim + 15) / 16);
        const int steps = delta_steps(dim);
        delta_f32x4* w = (delta_f32x4*)block_scratch;                   // (in units of four floats)
        delta_f32x4* q = w + rows * 4 * steps;
        delta_f32x4* kt = q + rows * 4 * steps;
        delta_f32x4* u = kt + rows * 4 * steps;
        delta_f32x4* p = u + rows * 4 * slices;
        float* gc = (float*)(p + rows * (DELTA_BLOCK / 4));
#define DELTA_BLOCKS(KK)                                                                                                  \
        do {                                                                                                              \
            hipLaunchKernelGGL((delta_block_solve_kernel<KK>), dim3((unsigned)(n_units * heads)), dim3(256), 0, stream, qn, kn, vf, decay, \
                               beta, units, heads, kv_heads, dim, vdim, gc, w, q, u, p, kt);                                  \
            hipLaunchKernelGGL((delta_block_scan_kernel<KK>), dim3((unsigned)(slices * n_chains * heads)), dim3(256), 0, stream, gc, w, q,   \
                               u, p, kt, o_raw, s_state, units, chains, (int)n_chains, seq_starts, state_slots, heads, dim,           \
                               vdim);                                                                                     \
        } while (0)
        if (steps == 2) DELTA_BLOCKS(2); else if (steps == 4) DELTA_BLOCKS(4); else if (steps == 8) DELTA_BLOCKS(8); else DELTA_BLOCKS(16);
#undef DELTA_BLOCKS
    }
    hipLaunchKernelGGL((delta_finish_kernel<elem_t, true>), dim3((unsigned)left, (unsigned)heads), dim3(NVA_WAVE), 0, stream, o_raw,
                       pr + channels, stride, norm_w, eps, (elem_t*)out, out_stride, heads, vdim, first);
    return nva_check_launch("head_delta");
}

NVA_DEFINE_LAST_ERROR(nva_delta)
