// Linear attentions whose state forgets by a decay that depends on the token, after their projections: two rules over a
// float state S [D, DV] per head and request that starts at zero.  q is multiplied by D^-1/2.
//
//   linear  S <- diag(a) S + k v^T;  o = S^T q;  a = sigmoid(z)^(1/tau) per head and key channel;
//           y = o / sqrt(mean(o^2) + eps) * w * silu(gate)           per head, w [DV] shared by the heads
//   matrix  i = c tanh(zi / c),  f = logsigmoid(c tanh(zf / c))      one number per head each
//           m' = max(f + m, i);  S <- exp(f + m - m') S + exp(i - m') k v^T;  n <- exp(f + m - m') n + exp(i - m') k
//           o = S^T q / (max(|n . q|, exp(-m')) + 1e-6);             m starts at 0, n [D] at zero
//           y = o / sqrt(mean(o^2) + eps) * w * sigmoid(gate)        the norm per head, w over all heads' channels
//
// The projections' row is [q | k | v | gate] (linear: and behind them the decay's low-rank input).  Everything after the
// projections is float; y is rounded once.  The step's metadata is read on the device only.
//
// Single tokens: memory_walk_kernel, a workgroup per (request, head), everything from the gates to the output in one
// pass over the state, which is read once and written once.  The same kernel walks portions token by token where the sizes
// are beyond what the next takes.
//
// Portions: in chunks of 16 tokens on the matrix cores (float products, v_mfma_f32_16x16x4_f32).  Within a chunk let P_t be
// the sum of log a over its tokens up to t (linear; per channel), P the whole chunk's.  With S the state before the chunk,
//     o_t = S^T (q_t exp(P_t)) + sum_{s <= t} A_ts v_s,    A_ts = sum_d q_td k_sd exp(P_td - P_sd)
//     S'  = diag(exp(P)) S + sum_s (k_s exp(P - P_s)) v_s^T
// and for the matrix rule, with b the running sum of f, e_s = i_s - b_s and M_t = max(M before the portion, max_{s <= t} e_s)
// (so that m_t = b_t + M_t; e and M are kept in double, made by memory_gates_kernel for a whole portion at once),
//     o_t = exp(M_c - M_t) S^T q_t + sum_{s <= t} exp(e_s - M_t) (q_t . k_s) v_s,     M_c the maximum before the chunk
//     S'  = exp(M_c - M_end) S + sum_s exp(e_s - M_end) k_s v_s^T
// No exponent of these is positive.  In the linear rule A's factors exp(P_t) and exp(-P_s) are applied to q and k apart as long
// as no channel of 16 forgets more than exp(-MEM_APART) in a chunk; where one does, that group of channels is summed pair by pair.
//
// A workgroup takes a unit (a run of chunks of one request) and a head; a wave 16 value channels, whose part of S it keeps in
// accumulators: register r of tile j holds, in lane group g = lane / 16, row 16 j + 4 g + r, which is how the product with q
// takes it as its right operand.  Long portions are cut into units that run side by side: memory_block_kernel without
// outputs leaves every unit's end state from zero, memory_scan_kernel turns these into the units' states at their starts, and
// memory_block_kernel with outputs runs each from there; the last unit leaves the request's new state.
#include "common.h"

enum { MEM_LINEAR = 0, MEM_MATRIX = 1 };
#define MEM_APART 12.f

typedef __attribute__((ext_vector_type(4))) float mem_f32x4;

struct MemoryArgs {
    const void* proj; int64_t stride;                       // rows [q | k | v | gate (| low)]
    const float* z; int64_t z_first;                        // linear: logits [tokens from z_first on][H D], without the bias, or null
    const void* a2; int rank;                               // linear: [H D, rank]: the logits' second step, for single tokens
    const float* gates; int splits; int64_t split_stride;   // matrix: [splits][tokens][2 H] = [i | f], without the bias
    const float* bias;                                      // linear [H D], matrix [2 H]
    const float* norm_w; float eps, par;                    // par: 1 / tau, or the gates' cap
    float* s_state; float* n_state; float* m_state;
    const int32_t* cu_seqlens_q; const int32_t* seq_starts; const int32_t* state_slots;
    void* out; int64_t out_stride;
    int heads, dim, vdim;
    float scale;                                            // D^-1/2
    // portions
    const int32_t* units; const int32_t* chains;            // [n][4]: request, first token of the step, tokens, kind; [n][4]: first unit, units, request, 0
    float* unit_states; float* unit_decay;                  // [units][H][D DV (+ D)], [units][H][D]
    int64_t tokens;
    double* e; double* M; float* m; float* m_start;         // matrix: [H][tokens] three times, [requests][H]
};
enum { MEM_UNIT_ONLY = 0, MEM_UNIT_MORE = 1, MEM_UNIT_LAST = 2 };

// log sigmoid(x) = min(x, 0) - log(1 + e), e = exp(-|x|).  The bfloat16 build takes the fast exponential and logarithm, and what
// the rounding of u = 1 + e lost of e back in: log(1 + e) = log u + (e - (u - 1)) / u to first order.
__device__ __forceinline__ float mem_log_sigmoid(float x) {
#if defined(NVA_F32)
    return fminf(x, 0.f) - log1pf(expf(-fabsf(x)));
#else
    const float e = __expf(-fabsf(x)), u = 1.f + e;
    return fminf(x, 0.f) - (__logf(u) + (e - (u - 1.f)) * __frcp_rn(u));
#endif
}
__device__ __forceinline__ float mem_sigmoid(float x) { return 1.f / (1.f + nva_exp(-x)); }
template <int KIND> __device__ __forceinline__ float mem_gate(float g) { return KIND == MEM_LINEAR ? g * mem_sigmoid(g) : mem_sigmoid(g); }

// The capped gates of a (token, head): i and f = logsigmoid(capped).
__device__ __forceinline__ void mem_gates(const MemoryArgs& a, int64_t tok, int h, float& gi, float& gf) {
    float zi = a.bias[h], zf = a.bias[a.heads + h];
    const float* p = a.gates + tok * 2 * a.heads + h;
#pragma unroll 8
    for (int s = 0; s < a.splits; ++s) {
        zi += p[s * a.split_stride];
        zf += p[s * a.split_stride + a.heads];
    }
    gi = a.par * tanhf(zi / a.par);
    gf = mem_log_sigmoid(a.par * tanhf(zf / a.par));
}

// ---------------------------------------------------------------------------- token by token
#define MEM_WALK_MAX 512
#define MEM_WALK_ROWS 8              // rows of S that a thread asks for at once
// LDS: q, k, decay [D] each, o [DV], partial sums [threads * VEC].
template <typename T, int KIND, int VEC>
__global__ void __launch_bounds__(MEM_WALK_MAX)
memory_walk_kernel(const MemoryArgs a, int first_seq) {
    extern __shared__ __attribute__((aligned(16))) float lds[];
    __shared__ float scratch[16];
    const int h = blockIdx.x, seq = first_seq + blockIdx.y, tid = threadIdx.x, nt = blockDim.x;
    const int D = a.dim, DV = a.vdim, H = a.heads;
    const int DP = (D + 3) / 4 * 4, DVP = (DV + 3) / 4 * 4;
    float* const part_s = lds;                               // [threads * VEC]
    float* const q_s = part_s + nt * VEC;
    float* const k_s = q_s + DP;
    float* const a_s = k_s + DP;
    float* const o_s = a_s + DP;
    const int64_t tok0 = a.cu_seqlens_q[seq];
    const int n_tok = a.cu_seqlens_q[seq + 1] - (int)tok0;
    const int64_t slot = a.state_slots[seq];
    bool fresh = a.seq_starts[seq] <= 0;
    const T* proj = static_cast<const T*>(a.proj);
    float* const S = a.s_state + (slot * H + h) * D * DV;
    float* const N = KIND == MEM_MATRIX ? a.n_state + (slot * H + h) * D : nullptr;
    float m = KIND == MEM_MATRIX && !fresh ? a.m_state[slot * H + h] : 0.f;
    const int cols = DV / VEC;                               // (VEC divides DV: the launcher's choice)
    const int tx_n = min(cols, nt), ty_n = nt / tx_n;
    const int tx = tid % tx_n, ty = tid / tx_n;
    const int64_t qk = (int64_t)H * D, vv = (int64_t)H * DV;
    for (int j = 0; j < n_tok; ++j) {
        const int64_t tok = tok0 + j;
        const T* row = proj + tok * a.stride;
        float keep = 1.f, write = 1.f;
        if (KIND == MEM_MATRIX) {
            float gi, gf;
            mem_gates(a, tok, h, gi, gf);
            const float m_new = fmaxf(gf + m, gi);
            keep = expf(gf + m - m_new);
            write = expf(gi - m_new);
            m = m_new;
        }
        float nq = 0.f;
        for (int d = tid; d < D; d += nt) {
            const float qv = to_float(row[(int64_t)h * D + d]) * a.scale, kv = to_float(row[qk + (int64_t)h * D + d]);
            q_s[d] = qv;
            if (KIND == MEM_MATRIX) {
                k_s[d] = write * kv;
                const float nv = (fresh ? 0.f : keep * N[d]) + write * kv;
                N[d] = nv;
                nq += nv * qv;
            } else {
                k_s[d] = kv;
                const int64_t c = (int64_t)h * D + d;
                float z = a.bias[c];
                if (a.a2) {
                    const T* low = row + 2 * qk + 2 * vv;
                    const T* w = static_cast<const T*>(a.a2) + c * a.rank;
                    float sum = 0.f;
#pragma unroll 8
                    for (int r = 0; r < a.rank; ++r) sum += to_float(low[r]) * to_float(w[r]);
                    z += sum;
                } else {
                    z += a.z[(tok - a.z_first) * qk + c];
                }
                a_s[d] = expf(mem_log_sigmoid(z) * a.par);
            }
        }
        if (KIND == MEM_MATRIX) nq = block_sum(nq, scratch);
        __syncthreads();
        for (int c0 = 0; c0 < cols; c0 += tx_n) {
            const int c = c0 + tx;
            const bool has = c < cols && ty < ty_n;
            float v[VEC], o[VEC];
#pragma unroll
            for (int e = 0; e < VEC; ++e) {
                v[e] = has ? to_float(row[2 * qk + (int64_t)h * DV + c * VEC + e]) : 0.f;
                o[e] = 0.f;
            }
            if (has) {
                for (int d0 = ty; d0 < D; d0 += ty_n * MEM_WALK_ROWS) {
                    float s[MEM_WALK_ROWS][VEC];
#pragma unroll
                    for (int u = 0; u < MEM_WALK_ROWS; ++u) {
                        const float* p = S + (int64_t)min(d0 + u * ty_n, D - 1) * DV + c * VEC;
                        if (fresh) {
#pragma unroll
                            for (int e = 0; e < VEC; ++e) s[u][e] = 0.f;
                        } else if (VEC == 4) {
                            const float4 x = *reinterpret_cast<const float4*>(p);
                            s[u][0] = x.x; s[u][VEC > 1 ? 1 : 0] = x.y; s[u][VEC > 2 ? 2 : 0] = x.z; s[u][VEC > 3 ? 3 : 0] = x.w;
                        } else {
#pragma unroll
                            for (int e = 0; e < VEC; ++e) s[u][e] = p[e];
                        }
                    }
#pragma unroll
                    for (int u = 0; u < MEM_WALK_ROWS; ++u) {
                        const int d = d0 + u * ty_n;
                        if (d >= D) continue;
                        const float keep_d = KIND == MEM_MATRIX ? keep : a_s[d], kd = k_s[d], qd = q_s[d];
#pragma unroll
                        for (int e = 0; e < VEC; ++e) {
                            s[u][e] = keep_d * s[u][e] + kd * v[e];
                            o[e] += s[u][e] * qd;
                        }
                        float* p = S + (int64_t)d * DV + c * VEC;
                        if (VEC == 4) *reinterpret_cast<float4*>(p) = make_float4(s[u][0], s[u][VEC > 1 ? 1 : 0], s[u][VEC > 2 ? 2 : 0], s[u][VEC > 3 ? 3 : 0]);
                        else
#pragma unroll
                            for (int e = 0; e < VEC; ++e) p[e] = s[u][e];
                    }
                }
            }
            if (ty < ty_n)
#pragma unroll
                for (int e = 0; e < VEC; ++e) part_s[(ty * tx_n + tx) * VEC + e] = o[e];
            __syncthreads();
            for (int x = tid; x < tx_n * VEC; x += nt) {
                if (c0 * VEC + x < DV) {
                    float sum = 0.f;
                    for (int y = 0; y < ty_n; ++y) sum += part_s[y * tx_n * VEC + x];
                    o_s[c0 * VEC + x] = sum;
                }
            }
            __syncthreads();
        }
        const float div = KIND == MEM_MATRIX ? 1.f / (fmaxf(fabsf(nq), expf(-m)) + 1e-6f) : 1.f;
        float ss = 0.f;
        for (int c = tid; c < DV; c += nt) {
            const float x = o_s[c] * div;
            ss += x * x;
        }
        ss = block_sum(ss, scratch);
        const float inv = rsqrtf(ss / (float)DV + a.eps);
        for (int c = tid; c < DV; c += nt) {
            const float gate = to_float(row[2 * qk + vv + (int64_t)h * DV + c]);
            const float w = a.norm_w[KIND == MEM_MATRIX ? h * DV + c : c];
            static_cast<T*>(a.out)[tok * a.out_stride + (int64_t)h * DV + c] = from_float<T>(o_s[c] * div * inv * w * mem_gate<KIND>(gate));
        }
        fresh = false;
        __syncthreads();                                     // (q, k, the decays and the sums are written again)
    }
    if (KIND == MEM_MATRIX && tid == 0) a.m_state[slot * H + h] = m;
}

// ---------------------------------------------------------------------------- the matrix rule's gates of a portion
// A workgroup per (portion, head): b, e and M of its tokens by scans over MEM_SCAN tokens at a time, in double.
#define MEM_SCAN 1024
__device__ __forceinline__ double mem_shfl_up(double x, int by) {
    const unsigned long long u = __builtin_bit_cast(unsigned long long, x);
    const int lo = __shfl_up((int)(u & 0xffffffffull), by, NVA_WAVE), hi = __shfl_up((int)(u >> 32), by, NVA_WAVE);
    return __builtin_bit_cast(double, ((unsigned long long)(unsigned)hi << 32) | (unsigned)lo);
}

__global__ void __launch_bounds__(MEM_SCAN)
memory_gates_kernel(const MemoryArgs a, int first_seq) {
    __shared__ double wave_s[2][MEM_SCAN / NVA_WAVE];
    const int h = blockIdx.x, seq = first_seq + blockIdx.y, tid = threadIdx.x, lane = tid % NVA_WAVE, wave = tid / NVA_WAVE;
    const int H = a.heads;
    const int64_t tok0 = a.cu_seqlens_q[seq];
    const int n = a.cu_seqlens_q[seq + 1] - (int)tok0;
    const int64_t slot = a.state_slots[seq];
    const float m0 = a.seq_starts[seq] > 0 ? a.m_state[slot * H + h] : 0.f;
    if (tid == 0) a.m_start[(int64_t)seq * H + h] = m0;
    double b_carry = 0.0, max_carry = (double)m0, m_last = 0.0;
    for (int t0 = 0; t0 < n; t0 += MEM_SCAN) {
        const int t = t0 + tid;
        float gi = 0.f, gf = 0.f;
        if (t < n) mem_gates(a, tok0 + t, h, gi, gf);
        double b = (double)gf;
#pragma unroll
        for (int by = 1; by < NVA_WAVE; by <<= 1) {
            const double x = mem_shfl_up(b, by);
            if (lane >= by) b += x;
        }
        __syncthreads();                                     // (the pass before has read the waves' sums and maxima)
        if (lane == NVA_WAVE - 1) wave_s[0][wave] = b;
        __syncthreads();
        double before = b_carry;
#pragma unroll
        for (int w = 0; w < MEM_SCAN / NVA_WAVE; ++w) {
            if (w < wave) before += wave_s[0][w];
            b_carry += wave_s[0][w];
        }
        b += before;
        const double e = t < n ? (double)gi - b : -1e300;
        double mx = e;
#pragma unroll
        for (int by = 1; by < NVA_WAVE; by <<= 1) {
            const double x = mem_shfl_up(mx, by);
            if (lane >= by) mx = fmax(mx, x);
        }
        if (lane == NVA_WAVE - 1) wave_s[1][wave] = mx;
        __syncthreads();
        double top = max_carry;
#pragma unroll
        for (int w = 0; w < MEM_SCAN / NVA_WAVE; ++w) {
            if (w < wave) top = fmax(top, wave_s[1][w]);
            max_carry = fmax(max_carry, wave_s[1][w]);
        }
        mx = fmax(mx, top);
        if (t < n) {
            const int64_t at = (int64_t)h * a.tokens + tok0 + t;
            a.e[at] = e;
            a.M[at] = mx;
            m_last = b + mx;
            a.m[at] = (float)m_last;
            if (t == n - 1) a.m_state[slot * H + h] = (float)m_last;
        }
    }
}

// ---------------------------------------------------------------------------- portions in chunks of 16 tokens
#define MEM_C 16
#define MEM_TS 20                    // row stride of a transposed key row and of a chunk's scores

// Waves of a workgroup: one for every 16 key channels (a wave prepares one such tile a chunk) and for every 16 value channels.
__host__ __device__ inline int mem_block_waves(int ndt, int vdim) { return ndt > (vdim + 15) / 16 ? ndt : (vdim + 15) / 16; }

__host__ __device__ inline int mem_block_lds_floats(int ndt, int waves, bool out) {
    const int dp = 16 * ndt;
    int n = dp * MEM_TS + 3 * dp + 2 * MEM_C + 4;            // keys, decays, n, the unit's logarithms, weights and factors
    if (out) n += MEM_C * (dp + 4) + waves * MEM_C * MEM_TS + MEM_C * MEM_TS + 2 * waves * MEM_C + 2 * MEM_C;
    return n;
}

template <typename T, int KIND, int NDT, bool OUT, int THREADS>
__global__ void __launch_bounds__(THREADS)
memory_block_kernel(const MemoryArgs a) {
    extern __shared__ __attribute__((aligned(16))) float lds[];
    __shared__ double e_s[MEM_C], M_s[MEM_C];
    constexpr int DP = 16 * NDT, QS = DP + 4;
    const int waves = blockDim.x / NVA_WAVE, wave = threadIdx.x / NVA_WAVE, lane = threadIdx.x % NVA_WAVE;
    const int i = lane & 15, g = lane >> 4, tid = threadIdx.x;
    float* const kT_s = lds;                                 // [DP][20]: keys times their decay to the chunk's end
    float* const dec_s = kT_s + DP * MEM_TS;                 // [DP]: the chunk's decays (linear)
    float* const n_s = dec_s + DP;                           // [DP] (matrix)
    float* const log_s = n_s + DP;                           // [DP]: the unit's log decays so far (linear, without outputs)
    float* const w_s = log_s + DP;                           // [16]: exp(e_s - M_end)
    float* const inter_s = w_s + MEM_C;                      // [16]: exp(M_c - M_t)
    float* const keep_s = inter_s + MEM_C;                   // [1] (+ 3)
    float* const q_s = keep_s + 4;                           // [16][QS]
    float* const part_s = q_s + MEM_C * QS;                  // [waves][16 * 20]: a wave's keys, then its part of the scores
    float* const a_s = part_s + waves * MEM_C * MEM_TS;      // [16][20]: the scores
    float* const red_s = a_s + MEM_C * MEM_TS;               // [waves][16]
    float* const qn_s = red_s + waves * MEM_C;               // [waves][16]
    float* const den_s = qn_s + waves * MEM_C;               // [16]
    float* const floor_s = den_s + MEM_C;                    // [16]: exp(-m_t)

    const int h = blockIdx.x;
    const int32_t* u = a.units + 4 * (int64_t)blockIdx.y;
    const int seq = u[0], n_tok = u[2], kind = u[3];
    const int64_t tok0 = u[1];
    if (!OUT && kind != MEM_UNIT_MORE) return;               // (a portion's last unit needs no end state from zero)
    const int D = a.dim, DV = a.vdim, H = a.heads;
    const int64_t qk = (int64_t)H * D, vv = (int64_t)H * DV;
    const int64_t q_off = (int64_t)h * D, k_off = qk + q_off, v_off = 2 * qk + (int64_t)h * DV, g_off = v_off + vv;
    const T* const proj = static_cast<const T*>(a.proj);
    const int c = 16 * wave + i, cc = min(c, DV - 1);        // this lane's value channel
    const bool has_c = c < DV, multiplies = 16 * wave < DV;  // (a wave beyond the value channels only prepares)
    const int d_own = 16 * wave + i, dc = min(d_own, D - 1); // the key channel it prepares
    const bool prepares = wave < NDT, has_d = d_own < D;
    const int64_t slot = a.state_slots[seq];
    const bool fresh = a.seq_starts[seq] <= 0;
    const int64_t state_floats = (int64_t)D * DV + (KIND == MEM_MATRIX ? D : 0);
    float* const s_unit = a.unit_states + ((int64_t)blockIdx.y * H + h) * state_floats;      // (not read for a portion of one unit)
    float* const s_slot = a.s_state + (slot * H + h) * (int64_t)D * DV;
    float* const n_slot = KIND == MEM_MATRIX ? a.n_state + (slot * H + h) * (int64_t)D : nullptr;

    // ---- a chunk's values, gates, queries, keys and decay logits: asked for a chunk ahead, kept as they were loaded
    T v_raw[4], g_raw[4], q_raw[4], k_raw[4];
    float z_raw[4];
    double e_raw = 0.0, M_raw = 0.0, M_end_raw = 0.0;
    float m_raw = 0.f;
    auto ask = [&](int t0) __attribute__((always_inline)) {
        const int64_t tok = tok0 + t0;
        const int last = n_tok - t0 - 1;                     // (a token beyond the unit reads the unit's last)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
            const int64_t tt = tok + min(4 * g + r, last);
            const T* row = proj + tt * a.stride;
            v_raw[r] = row[v_off + cc];
            if (OUT) g_raw[r] = row[g_off + cc];
            if (OUT) q_raw[r] = row[q_off + dc];
            k_raw[r] = row[k_off + dc];
            if (KIND == MEM_LINEAR) z_raw[r] = a.z[(tt - a.z_first) * qk + q_off + dc];
        }
        if (KIND == MEM_MATRIX) {
            const int64_t at = (int64_t)h * a.tokens + tok + min(i, last);
            e_raw = a.e[at];
            M_raw = a.M[at];
            M_end_raw = a.M[(int64_t)h * a.tokens + tok + min(MEM_C - 1, last)];
            if (OUT) m_raw = a.m[at];
        }
    };
    ask(0);

    // ---- the state at the unit's start
    const float* s_from = !OUT ? nullptr : kind != MEM_UNIT_ONLY ? s_unit : fresh ? nullptr : s_slot;
    const float* n_from = KIND == MEM_LINEAR || !s_from ? nullptr : kind != MEM_UNIT_ONLY ? s_unit + (int64_t)D * DV : n_slot;
    mem_f32x4 S[NDT];
    if (s_from) {
#pragma unroll
        for (int j = 0; j < NDT; ++j)
#pragma unroll
            for (int r = 0; r < 4; ++r) S[j][r] = s_from[(int64_t)min(16 * j + 4 * g + r, D - 1) * DV + cc];
    }
#pragma unroll
    for (int j = 0; j < NDT; ++j)
#pragma unroll
        for (int r = 0; r < 4; ++r)
            if (!s_from || !has_c || 16 * j + 4 * g + r >= D) S[j][r] = 0.f;
    for (int d = tid; d < DP; d += blockDim.x) {
        n_s[d] = KIND == MEM_MATRIX && n_from && d < D ? n_from[d] : 0.f;
        dec_s[d] = 1.f;
        log_s[d] = 0.f;
    }
    double M_before = 0.0;
    if (KIND == MEM_MATRIX)
        M_before = tok0 == a.cu_seqlens_q[seq] ? (double)a.m_start[(int64_t)seq * H + h] : a.M[(int64_t)h * a.tokens + tok0 - 1];
    const double M_unit = M_before;
    const float bias = KIND == MEM_LINEAR ? a.bias[q_off + dc] : 0.f;
    const float norm_w = OUT ? a.norm_w[KIND == MEM_MATRIX ? h * DV + cc : cc] : 0.f;
    __syncthreads();

    for (int t0 = 0; t0 < n_tok; t0 += MEM_C) {
        const int n = min(MEM_C, n_tok - t0);
        const int64_t tok = tok0 + t0;
        float v[4], gate[4], q[4], k[4], lg[4];
#pragma unroll
        for (int r = 0; r < 4; ++r) {
            const bool has = has_d && 4 * g + r < n;
            v[r] = has_c && 4 * g + r < n ? to_float(v_raw[r]) : 0.f;
            if (OUT) gate[r] = to_float(g_raw[r]);
            if (OUT) q[r] = has ? to_float(q_raw[r]) * a.scale : 0.f;
            k[r] = has ? to_float(k_raw[r]) : 0.f;
            if (KIND == MEM_LINEAR) lg[r] = has ? z_raw[r] + bias : 0.f;
        }
        const double M_end = M_end_raw, e_now = i < n ? e_raw : -1e300, M_now = M_raw;
        const float m_now = m_raw;
        if (t0 + MEM_C < n_tok) ask(t0 + MEM_C);
        if (KIND == MEM_MATRIX && tid < MEM_C) {
            e_s[tid] = e_now;
            M_s[tid] = M_now;
            w_s[tid] = expf((float)(e_now - M_end));         // (a token beyond the unit: zero)
            inter_s[tid] = expf((float)(M_before - M_now));
            if (OUT) floor_s[tid] = expf(-m_now);
            if (tid == 0) keep_s[0] = expf((float)(M_before - M_end));
        }
        // ---- queries, keys and decays: a wave prepares 16 key channels; a lane one channel and four tokens
        float* const mine_s = part_s + wave * MEM_C * MEM_TS;
        if (prepares) {
            mem_f32x4 score = {0.f, 0.f, 0.f, 0.f};
            float qn[4] = {0.f, 0.f, 0.f, 0.f};
            bool apart = true;
            if (KIND == MEM_LINEAR) {
#pragma unroll
                for (int r = 0; r < 4; ++r) lg[r] = has_d && 4 * g + r < n ? mem_log_sigmoid(lg[r]) * a.par : 0.f;
                // sums up to and including a token, and behind it to the chunk's end
                const float p0 = lg[0], p1 = p0 + lg[1], p2 = p1 + lg[2], p3 = p2 + lg[3];
                const float x0 = __shfl(p3, i, NVA_WAVE), x1 = __shfl(p3, i + 16, NVA_WAVE), x2 = __shfl(p3, i + 32, NVA_WAVE),
                            x3 = __shfl(p3, i + 48, NVA_WAVE);
                const float base = (g > 0 ? x0 : 0.f) + (g > 1 ? x1 : 0.f) + (g > 2 ? x2 : 0.f);
                const float after = (g < 1 ? x1 : 0.f) + (g < 2 ? x2 : 0.f) + (g < 3 ? x3 : 0.f);
                const float all = x0 + x1 + x2 + x3;
                const float P[4] = {base + p0, base + p1, base + p2, base + p3};
                const float B[4] = {after + lg[3] + lg[2] + lg[1], after + lg[3] + lg[2], after + lg[3], after};
                if (g == 0) dec_s[d_own] = nva_exp(all);
                if (!OUT && g == 0) log_s[d_own] += all;
                *reinterpret_cast<mem_f32x4*>(kT_s + d_own * MEM_TS + 4 * g) =
                    mem_f32x4{k[0] * nva_exp(B[0]), k[1] * nva_exp(B[1]), k[2] * nva_exp(B[2]), k[3] * nva_exp(B[3])};
                if (OUT) {
                    apart = __all(all > -MEM_APART);
#pragma unroll
                    for (int r = 0; r < 4; ++r) q_s[(4 * g + r) * QS + d_own] = q[r] * nva_exp(P[r]);
                    if (apart) {
#pragma unroll
                        for (int r = 0; r < 4; ++r) mine_s[(4 * g + r) * MEM_TS + i] = k[r] * nva_exp(-P[r]);
                    } else {
                        // a channel that forgets nearly everything within the chunk: pair by pair
                        for (int s = 0; s < n; ++s) {
                            const int from = i + 16 * (s >> 2);
                            float ks = k[0], Ps = P[0];
                            if ((s & 3) == 1) { ks = k[1]; Ps = P[1]; }
                            else if ((s & 3) == 2) { ks = k[2]; Ps = P[2]; }
                            else if ((s & 3) == 3) { ks = k[3]; Ps = P[3]; }
                            ks = __shfl(ks, from, NVA_WAVE);
                            Ps = __shfl(Ps, from, NVA_WAVE);
#pragma unroll
                            for (int r = 0; r < 4; ++r) {
                                float x = 4 * g + r >= s ? q[r] * ks * nva_exp(fminf(P[r] - Ps, 0.f)) : 0.f;
#pragma unroll
                                for (int by = 1; by < 16; by <<= 1) x += __shfl_xor(x, by, NVA_WAVE);
                                if (i == s) score[r] += x;
                            }
                        }
                    }
                }
            } else {
                *reinterpret_cast<mem_f32x4*>(kT_s + d_own * MEM_TS + 4 * g) = mem_f32x4{k[0], k[1], k[2], k[3]};
                if (OUT) {
                    const float nd = n_s[d_own];
#pragma unroll
                    for (int r = 0; r < 4; ++r) {
                        q_s[(4 * g + r) * QS + d_own] = q[r];
                        mine_s[(4 * g + r) * MEM_TS + i] = k[r];
                        qn[r] = q[r] * nd;
                    }
                }
            }
            if (OUT) {
                // the tile's part of the scores (what the wave's lanes wrote, read by its other lanes)
                __builtin_amdgcn_wave_barrier();
                asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");
                if (apart) {
                    const mem_f32x4 qa = *reinterpret_cast<const mem_f32x4*>(q_s + i * QS + 16 * wave + 4 * g);
                    const mem_f32x4 kb = *reinterpret_cast<const mem_f32x4*>(mine_s + i * MEM_TS + 4 * g);
#pragma unroll
                    for (int r = 0; r < 4; ++r) score = __builtin_amdgcn_mfma_f32_16x16x4f32(qa[r], kb[r], score, 0, 0, 0);
                }
                asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");
                __builtin_amdgcn_wave_barrier();
#pragma unroll
                for (int r = 0; r < 4; ++r) mine_s[(4 * g + r) * 17 + i] = score[r];
                if (KIND == MEM_MATRIX) {
#pragma unroll
                    for (int r = 0; r < 4; ++r) {
#pragma unroll
                        for (int by = 1; by < 16; by <<= 1) qn[r] += __shfl_xor(qn[r], by, NVA_WAVE);
                        if (i == 0) qn_s[wave * MEM_C + 4 * g + r] = qn[r];
                    }
                }
            }
        }
        __syncthreads();
        // ---- the scores added up over the waves, with their weights; the matrix rule's divisor
        if (OUT) {
            for (int idx = tid; idx < MEM_C * MEM_C; idx += blockDim.x) {
                const int t = idx >> 4, s = idx & 15;
                float x = 0.f;
#pragma unroll
                for (int w = 0; w < NDT; ++w) x += part_s[w * MEM_C * MEM_TS + t * 17 + s];
                if (s > t || t >= n) x = 0.f;
                if (KIND == MEM_MATRIX) {
                    x = s > t || t >= n ? 0.f : x * expf((float)(e_s[s] - M_s[t]));
                    float sum = x;
#pragma unroll
                    for (int by = 1; by < 16; by <<= 1) sum += __shfl_xor(sum, by, NVA_WAVE);
                    if (s == 0) {
                        float nq = 0.f;
#pragma unroll
                        for (int w = 0; w < NDT; ++w) nq += qn_s[w * MEM_C + t];
                        sum += inter_s[t] * nq;
                        den_s[t] = t < n ? 1.f / (fmaxf(fabsf(sum), floor_s[t]) + 1e-6f) : 0.f;
                    }
                }
                a_s[t * MEM_TS + s] = x;
            }
        }
        // ---- what the state gives, and the state behind the chunk
        mem_f32x4 o = {0.f, 0.f, 0.f, 0.f};
        const float keep = KIND == MEM_MATRIX ? keep_s[0] : 1.f;
        if (multiplies) {
            float vw[4];
#pragma unroll
            for (int r = 0; r < 4; ++r) vw[r] = KIND == MEM_MATRIX ? v[r] * w_s[4 * g + r] : v[r];
#pragma unroll
            for (int j = 0; j < NDT; ++j) {
                if (OUT) {
                    const mem_f32x4 qa = *reinterpret_cast<const mem_f32x4*>(q_s + i * QS + 16 * j + 4 * g);
#pragma unroll
                    for (int r = 0; r < 4; ++r) o = __builtin_amdgcn_mfma_f32_16x16x4f32(qa[r], S[j][r], o, 0, 0, 0);
                }
                if (KIND == MEM_LINEAR) {
                    const mem_f32x4 dec = *reinterpret_cast<const mem_f32x4*>(dec_s + 16 * j + 4 * g);
#pragma unroll
                    for (int r = 0; r < 4; ++r) S[j][r] *= dec[r];
                } else {
#pragma unroll
                    for (int r = 0; r < 4; ++r) S[j][r] *= keep;
                }
                const mem_f32x4 ka = *reinterpret_cast<const mem_f32x4*>(kT_s + (16 * j + i) * MEM_TS + 4 * g);
#pragma unroll
                for (int r = 0; r < 4; ++r) S[j] = __builtin_amdgcn_mfma_f32_16x16x4f32(ka[r], vw[r], S[j], 0, 0, 0);
            }
        }
        if (KIND == MEM_MATRIX) {
#pragma unroll
            for (int r = 0; r < 4; ++r) o[r] *= inter_s[4 * g + r];
            for (int d = tid; d < DP; d += blockDim.x) {
                float x = keep * n_s[d];
#pragma unroll
                for (int s = 0; s < MEM_C; ++s) x += w_s[s] * kT_s[d * MEM_TS + s];
                n_s[d] = x;
            }
            M_before = M_end;
        }
        __syncthreads();
        if (OUT) {
            // ---- the chunk's own tokens, the norm over the head's channels, the gate
            const mem_f32x4 sa = *reinterpret_cast<const mem_f32x4*>(a_s + i * MEM_TS + 4 * g);
#pragma unroll
            for (int r = 0; r < 4; ++r) o = __builtin_amdgcn_mfma_f32_16x16x4f32(sa[r], v[r], o, 0, 0, 0);
#pragma unroll
            for (int r = 0; r < 4; ++r) {
                if (KIND == MEM_MATRIX) o[r] *= den_s[4 * g + r];
                float x = o[r] * o[r];                       // (a channel beyond the head's is zero)
#pragma unroll
                for (int by = 1; by < 16; by <<= 1) x += __shfl_xor(x, by, NVA_WAVE);
                if (i == 0) red_s[wave * MEM_C + 4 * g + r] = x;
            }
            __syncthreads();
            mem_f32x4 ss = {0.f, 0.f, 0.f, 0.f};
            for (int x = 0; x < waves; ++x) ss += *reinterpret_cast<const mem_f32x4*>(red_s + x * MEM_C + 4 * g);
#pragma unroll
            for (int r = 0; r < 4; ++r) {
                const int t = 4 * g + r;
                const float inv = rsqrtf(ss[r] / (float)DV + a.eps);
                if (t < n && has_c)
                    static_cast<T*>(a.out)[(tok + t) * a.out_stride + (int64_t)h * DV + c] = from_float<T>(o[r] * inv * norm_w * mem_gate<KIND>(gate[r]));
            }
        }
    }
    // ---- the state behind the unit
    float* const s_to = !OUT ? s_unit : kind == MEM_UNIT_MORE ? nullptr : s_slot;
    float* const n_to = KIND == MEM_LINEAR || !s_to ? nullptr : OUT ? n_slot : s_unit + (int64_t)D * DV;
    if (s_to) {
#pragma unroll
        for (int j = 0; j < NDT; ++j)
#pragma unroll
            for (int r = 0; r < 4; ++r) {
                const int d = 16 * j + 4 * g + r;
                if (has_c && d < D) s_to[(int64_t)d * DV + c] = S[j][r];
            }
        if (n_to)
            for (int d = tid; d < D; d += blockDim.x) n_to[d] = n_s[d];
    }
    if (!OUT) {
        float* const dec = a.unit_decay + ((int64_t)blockIdx.y * H + h) * D;
        if (KIND == MEM_MATRIX) {
            const float x = expf((float)(M_unit - M_before));
            for (int d = tid; d < D; d += blockDim.x) dec[d] = x;
        } else {
            // (the last chunk's barriers lie between the sums and these reads)
            for (int d = tid; d < D; d += blockDim.x) dec[d] = expf(log_s[d]);
        }
    }
}

// The units' states at their starts from their end states from zero: E_0 the request's, E_(b+1) = decay_b E_b + state_b.
__global__ void __launch_bounds__(256)
memory_scan_kernel(const MemoryArgs a, int with_n) {
    const int32_t* ch = a.chains + 4 * (int64_t)blockIdx.z;
    const int first = ch[0], count = ch[1], seq = ch[2];
    const int h = blockIdx.y, D = a.dim, DV = a.vdim, H = a.heads;
    const int64_t whole = (int64_t)D * DV, total = whole + (with_n ? D : 0);
    const int64_t x = (int64_t)blockIdx.x * blockDim.x + threadIdx.x;
    if (x >= total) return;
    const int64_t slot = a.state_slots[seq];
    const int d = (int)(x < whole ? x / DV : x - whole);
    float E = 0.f;
    if (a.seq_starts[seq] > 0) E = x < whole ? a.s_state[(slot * H + h) * whole + x] : a.n_state[(slot * H + h) * (int64_t)D + d];
    float* p = a.unit_states + ((int64_t)first * H + h) * total + x;
    const float* dec = a.unit_decay + ((int64_t)first * H + h) * D + d;
    const int64_t step = (int64_t)H * total, dstep = (int64_t)H * D;
    for (int b0 = 0; b0 < count; b0 += 4) {
        float own[4], f[4];
#pragma unroll
        for (int b = 0; b < 4; ++b) {
            const int at = min(b0 + b, count - 1);           // (the last unit's own state and decay are not there, and not used)
            const bool use = at < count - 1;
            own[b] = use ? p[at * step] : 0.f;
            f[b] = use ? dec[at * dstep] : 0.f;
        }
#pragma unroll
        for (int b = 0; b < 4; ++b) {
            if (b0 + b >= count) break;
            p[(b0 + b) * step] = E;
            E = f[b] * E + own[b];
        }
    }
}

// ---------------------------------------------------------------------------- entry points
static int mem_ndt(int dim) { return dim <= 32 ? 2 : dim <= 64 ? 4 : dim <= 128 ? 8 : 16; }

// Whether portions run in chunks on the matrix cores for these sizes.
NVA_EXPORT int NVA_NAME(nva_memory_takes_blocks)(int dim, int vdim) { return dim <= 256 && vdim <= 256; }

template <int KIND, int NDT, bool OUT, int THREADS>
static int mem_launch_sized(const MemoryArgs& a, int waves, int64_t n_units, hipStream_t stream) {
    const size_t bytes = sizeof(float) * (size_t)mem_block_lds_floats(NDT, waves, OUT);
    auto kernel = memory_block_kernel<elem_t, KIND, NDT, OUT, THREADS>;
    static bool raised = false;
    if (!raised && bytes > 48 * 1024) {
        if (hipFuncSetAttribute((const void*)kernel, hipFuncAttributeMaxDynamicSharedMemorySize, 128 * 1024) != hipSuccess)
            return nva_fail("memory: cannot have %zu bytes of LDS", bytes);
        raised = true;
    }
    hipLaunchKernelGGL(kernel, dim3((unsigned)a.heads, (unsigned)n_units), dim3(waves * NVA_WAVE), bytes, stream, a);
    return nva_check_launch("memory blocks");
}

template <int KIND, int NDT, bool OUT>
static int mem_launch_block(const MemoryArgs& a, int64_t n_units, hipStream_t stream) {
    const int waves = mem_block_waves(NDT, a.vdim);          // (16 at most)
    return waves <= 8 ? mem_launch_sized<KIND, NDT, OUT, 512>(a, waves, n_units, stream)
                      : mem_launch_sized<KIND, NDT, OUT, 1024>(a, waves, n_units, stream);
}

template <int KIND, bool OUT>
static int mem_block(const MemoryArgs& a, int64_t n_units, hipStream_t stream) {
    switch (mem_ndt(a.dim)) {
        case 2: return mem_launch_block<KIND, 2, OUT>(a, n_units, stream);
        case 4: return mem_launch_block<KIND, 4, OUT>(a, n_units, stream);
        case 8: return mem_launch_block<KIND, 8, OUT>(a, n_units, stream);
        default: return mem_launch_block<KIND, 16, OUT>(a, n_units, stream);
    }
}

template <int KIND>
static int mem_run(MemoryArgs a, int64_t seqs, int64_t tokens, int64_t singles, int64_t n_units, int64_t n_chains, hipStream_t stream) {
    if (tokens == 0) return 0;
    const int64_t qk = (int64_t)a.heads * a.dim, vv = (int64_t)a.heads * a.vdim;
    if (tokens < 0 || seqs <= 0 || seqs > 65535 || singles < 0 || singles > seqs || a.heads <= 0 || a.heads > 65535 || a.dim <= 0 ||
        a.dim > 4096 || a.vdim <= 0 || a.vdim > 8192)
        return nva_fail("memory: bad sizes tokens=%lld requests=%lld heads=%d dim=%d vdim=%d", (long long)tokens, (long long)seqs, a.heads, a.dim, a.vdim);
    if (!a.proj || !a.bias || !a.norm_w || !a.s_state || !a.cu_seqlens_q || !a.seq_starts || !a.state_slots || !a.out ||
        a.stride < 2 * qk + 2 * vv + a.rank || a.out_stride < vv)
        return nva_fail("memory: a tensor is missing or too narrow");
    if (KIND == MEM_MATRIX && (!a.gates || a.splits <= 0 || !a.n_state || !a.m_state)) return nva_fail("memory: the gates or their state are missing");
    if (KIND == MEM_LINEAR && !a.a2 && !a.z) return nva_fail("memory: the decay's logits are missing");
    a.scale = 1.f / sqrtf((float)a.dim);
    a.tokens = tokens;
    const bool blocks = n_units > 0;
    if (blocks) {
        if (a.dim > 256 || a.vdim > 256 || !a.units || n_units > 65535 || n_chains < 0 || n_chains > 65535 ||
            (n_chains && (!a.chains || !a.unit_states || !a.unit_decay)))
            return nva_fail("memory: portions of heads of %d and %d channels do not run in blocks, or their tensors are missing", a.dim, a.vdim);
        if (KIND == MEM_LINEAR && !a.z) return nva_fail("memory: the portions' decay logits are missing");
        if (KIND == MEM_MATRIX && (!a.e || !a.M || !a.m || !a.m_start)) return nva_fail("memory: room for the portions' gates is missing");
    }
    auto walk = [&](const MemoryArgs& w, int64_t first, int64_t count) -> int {
        const int nt = (int64_t)w.dim * w.vdim >= 8192 ? 512 : 256;
        const bool four = w.vdim % 4 == 0;                  // (a state's rows then start at whole float4s)
        const size_t bytes = sizeof(float) * (size_t)(nt * (four ? 4 : 1) + 3 * ((w.dim + 3) / 4 * 4) + (w.vdim + 3) / 4 * 4);
        if (bytes > 120 * 1024) return nva_fail("memory: heads of %d and %d channels need %zu bytes of LDS", w.dim, w.vdim, bytes);
        auto kernel = four ? memory_walk_kernel<elem_t, KIND, 4> : memory_walk_kernel<elem_t, KIND, 1>;
        if (bytes > 48 * 1024 && hipFuncSetAttribute((const void*)kernel, hipFuncAttributeMaxDynamicSharedMemorySize, 128 * 1024) != hipSuccess)
            return nva_fail("memory: cannot have %zu bytes of LDS", bytes);
        hipLaunchKernelGGL(kernel, dim3((unsigned)w.heads, (unsigned)count), dim3(nt), bytes, stream, w, (int)first);
        return nva_check_launch("memory walk");
    };
    const int64_t walked = blocks ? singles : seqs;
    if (walked > 0) {
        MemoryArgs w = a;
        if (KIND == MEM_LINEAR && w.a2) w.z = nullptr;
        if (KIND == MEM_LINEAR && !w.a2 && w.z_first > 0) return nva_fail("memory: the single tokens' decay logits are missing");
        const int rc = walk(w, 0, walked);
        if (rc) return rc;
    }
    if (!blocks) return 0;
    if (KIND == MEM_MATRIX) {
        hipLaunchKernelGGL(memory_gates_kernel, dim3((unsigned)a.heads, (unsigned)(seqs - singles)), dim3(MEM_SCAN), 0, stream, a, (int)singles);
        const int rc = nva_check_launch("memory gates");
        if (rc) return rc;
    }
    if (n_chains) {
        int rc = mem_block<KIND, false>(a, n_units, stream);
        if (rc) return rc;
        const int64_t total = (int64_t)a.dim * a.vdim + (KIND == MEM_MATRIX ? a.dim : 0);
        hipLaunchKernelGGL(memory_scan_kernel, dim3((unsigned)((total + 255) / 256), (unsigned)a.heads, (unsigned)n_chains), dim3(256), 0, stream,
                           a, KIND == MEM_MATRIX ? 1 : 0);
        rc = nva_check_launch("memory scan");
        if (rc) return rc;
    }
    return mem_block<KIND, true>(a, n_units, stream);
}

// The linear rule.  Requests [0, singles) bring one token each.  z: float logits [tokens - z_first, H D] of the tokens from
// z_first on (null: every token's are made from the row's low-rank input and a2 [H D, rank]).  n_units > 0: the requests
// from `singles` on run in blocks (units [n][4], chains [n][4]; unit_states, unit_decay as in MemoryArgs where there are chains).
NVA_EXPORT int NVA_NAME(nva_gated_linear)(const void* proj, int64_t stride, const float* z, int64_t z_first, const void* a2, int rank,
                                          const float* bias, const float* norm_w, float eps, float inv_tau, float* s_state,
                                          const int32_t* cu_seqlens_q, const int32_t* seq_starts, const int32_t* state_slots, void* out,
                                          int64_t out_stride, int64_t seqs, int64_t tokens, int64_t singles, int heads, int dim, int vdim,
                                          const int32_t* units, int64_t n_units, const int32_t* chains, int64_t n_chains,
                                          float* unit_states, float* unit_decay, hipStream_t stream) {
    MemoryArgs a = {};
    a.proj = proj; a.stride = stride; a.z = z; a.z_first = z_first; a.a2 = a2; a.rank = rank; a.bias = bias; a.norm_w = norm_w;
    a.eps = eps; a.par = inv_tau; a.s_state = s_state; a.cu_seqlens_q = cu_seqlens_q; a.seq_starts = seq_starts; a.state_slots = state_slots;
    a.out = out; a.out_stride = out_stride; a.heads = heads; a.dim = dim; a.vdim = vdim; a.units = units; a.chains = chains;
    a.unit_states = unit_states; a.unit_decay = unit_decay;
    return mem_run<MEM_LINEAR>(a, seqs, tokens, singles, n_units, n_chains, stream);
}

// The matrix rule.  gates: float partial sums [splits][tokens][2 H] = [i | f]; e, M: double [H, tokens], m: float [H, tokens],
// m_start: float [requests, H], scratch of the portions' gates.
NVA_EXPORT int NVA_NAME(nva_matrix_memory)(const void* proj, int64_t stride, const float* gates, int splits, int64_t split_stride,
                                           const float* bias, const float* norm_w, float eps, float cap, float* s_state, float* n_state,
                                           float* m_state, const int32_t* cu_seqlens_q, const int32_t* seq_starts,
                                           const int32_t* state_slots, void* out, int64_t out_stride, int64_t seqs, int64_t tokens,
                                           int64_t singles, int heads, int dim, int vdim, const int32_t* units, int64_t n_units,
                                           const int32_t* chains, int64_t n_chains, float* unit_states, float* unit_decay, double* e,
                                           double* M, float* m, float* m_start, hipStream_t stream) {
    MemoryArgs a = {};
    a.proj = proj; a.stride = stride; a.gates = gates; a.splits = splits; a.split_stride = split_stride; a.bias = bias; a.norm_w = norm_w;
    a.eps = eps; a.par = cap; a.s_state = s_state; a.n_state = n_state; a.m_state = m_state; a.cu_seqlens_q = cu_seqlens_q;
    a.seq_starts = seq_starts; a.state_slots = state_slots; a.out = out; a.out_stride = out_stride; a.heads = heads; a.dim = dim;
    a.vdim = vdim; a.units = units; a.chains = chains; a.unit_states = unit_states; a.unit_decay = unit_decay;
    a.e = e; a.M = M; a.m = m; a.m_start = m_start;
    if (!(cap > 0.f)) return nva_fail("memory: a gate cap of %f", cap);
    return mem_run<MEM_MATRIX>(a, seqs, tokens, singles, n_units, n_chains, stream);
}

NVA_DEFINE_LAST_ERROR(nva_memory)
