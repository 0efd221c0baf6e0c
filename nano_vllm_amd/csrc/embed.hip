// Row gather: out[t, :] = table[ids[t], :].  Serves the token embedding
// (nanovllm/layers/embed_head.py:38) and the selection of the rows whose logits are wanted
// (embed_head.py:59-60).  An id outside [0, rows) yields a row of zeros and raises the error
// flag, which the host reads after the step; ids that come from the host are checked there.
#include "common.h"

template <typename T>
__global__ void __launch_bounds__(256)
gather_rows_kernel(const T* __restrict__ table, int64_t table_stride, int64_t table_rows,
                   const int32_t* __restrict__ ids, T* __restrict__ out, int64_t out_stride, int width,
                   int vec, int32_t* error_flag) {
    const int64_t t = blockIdx.x;
    const int64_t id = ids[t];
    const bool ok = id >= 0 && id < table_rows;
    if (!ok && threadIdx.x == 0 && error_flag) atomicOr(error_flag, 1);
    const T* src = table + (ok ? id : 0) * table_stride;
    T* dst = out + t * out_stride;
    if (vec) {
        typedef __attribute__((ext_vector_type(4))) uint32_t u32x4;
        const int per = 16 / sizeof(T);
        const u32x4 zero = {0, 0, 0, 0};
        for (int i = threadIdx.x * per; i < width; i += blockDim.x * per)
            *reinterpret_cast<u32x4*>(dst + i) = ok ? *reinterpret_cast<const u32x4*>(src + i) : zero;
    } else {
        for (int i = threadIdx.x; i < width; i += blockDim.x) dst[i] = ok ? src[i] : from_float<T>(0.f);
    }
}

NVA_EXPORT int NVA_NAME(nva_gather_rows)(const void* table, int64_t table_stride, int64_t table_rows,
                                         const int32_t* ids, void* out, int64_t out_stride,
                                         int64_t count, int width, int32_t* error_flag, hipStream_t stream) {
    if (count == 0) return 0;
    if (count < 0 || count > 0x7fffffff || width <= 0 || table_rows <= 0)
        return nva_fail("gather_rows: bad shape count=%lld width=%d rows=%lld", (long long)count, width,
                        (long long)table_rows);
    const int per = 16 / sizeof(elem_t);
    const int vec = width % per == 0 && table_stride % per == 0 && out_stride % per == 0 &&
                    nva_aligned(table, 16) && nva_aligned(out, 16);
    const int threads = width >= 2048 ? 256 : (width >= 512 ? 128 : 64);
    hipLaunchKernelGGL(gather_rows_kernel<elem_t>, dim3((unsigned)count), dim3(threads), 0, stream,
                       (const elem_t*)table, table_stride, table_rows, ids, (elem_t*)out, out_stride, width,
                       vec, error_flag);
    return nva_check_launch("gather_rows");
}

// x <- x * factor over a float tensor of rows `stride` apart (logits times a model's constant).
__global__ void scale_rows_kernel(float* __restrict__ x, int64_t stride, int64_t rows, int width, float factor) {
    const int64_t idx = (int64_t)blockIdx.x * blockDim.x + threadIdx.x;
    if (idx >= rows * width) return;
    float* p = x + (idx / width) * stride + idx % width;
    *p = *p * factor;
}

NVA_EXPORT int NVA_NAME(nva_scale_rows)(float* x, int64_t stride, int64_t rows, int width, float factor, hipStream_t stream) {
    if (rows == 0) return 0;
    if (rows < 0 || width <= 0 || stride < width || !x) return nva_fail("scale_rows: bad arguments");
    const int64_t total = rows * width;
    hipLaunchKernelGGL(scale_rows_kernel, dim3((unsigned)((total + 255) / 256)), dim3(256), 0, stream, x, stride, rows, width,
                       factor);
    return nva_check_launch("scale_rows");
}

// x <- cap * tanh(x / cap) over a float tensor of rows `stride` apart (logits capped smoothly), four entries a thread where
// rows and pointer allow.
__global__ void __launch_bounds__(256) softcap_rows_kernel(float* __restrict__ x, int64_t stride, int64_t rows, int width, float cap,
                                                           float inv) {
    const int64_t idx = (int64_t)blockIdx.x * blockDim.x + threadIdx.x;
    if (idx >= rows * width) return;
    float* p = x + (idx / width) * stride + idx % width;
    *p = cap * tanhf(*p * inv);
}
__global__ void __launch_bounds__(256) softcap_rows4_kernel(float* __restrict__ x, int64_t stride, int64_t rows, int width4, float cap,
                                                            float inv) {
    const int64_t idx = (int64_t)blockIdx.x * blockDim.x + threadIdx.x;
    if (idx >= rows * width4) return;
    float4* p = reinterpret_cast<float4*>(x + (idx / width4) * stride) + idx % width4;
    float4 v = *p;
    v.x = cap * tanhf(v.x * inv); v.y = cap * tanhf(v.y * inv);
    v.z = cap * tanhf(v.z * inv); v.w = cap * tanhf(v.w * inv);
    *p = v;
}

NVA_EXPORT int NVA_NAME(nva_softcap_rows)(float* x, int64_t stride, int64_t rows, int width, float cap, hipStream_t stream) {
    if (rows == 0) return 0;
    if (rows < 0 || width <= 0 || stride < width || !x || !(cap > 0.f)) return nva_fail("softcap_rows: bad arguments");
    const bool four = width % 4 == 0 && stride % 4 == 0 && nva_aligned(x, 16);
    const int64_t total = rows * (four ? width / 4 : width);
    if ((total + 255) / 256 > 0x7fffffff) return nva_fail("softcap_rows: too many entries");
    const dim3 grid((unsigned)((total + 255) / 256));
    if (four) hipLaunchKernelGGL(softcap_rows4_kernel, grid, dim3(256), 0, stream, x, stride, rows, width / 4, cap, 1.f / cap);
    else hipLaunchKernelGGL(softcap_rows_kernel, grid, dim3(256), 0, stream, x, stride, rows, width, cap, 1.f / cap);
    return nva_check_launch("softcap_rows");
}

// A float stream as a sum of learned rows:
//     out[t] = table[ids[t]] + bigram[row] + positions[p_t]            all sums float; bigram and positions may be absent
//     row = (before * mul_prev + ids[t] * mul_cur) mod buckets, before = the token before this one in its sequence, or
//     row = buckets for a sequence's first token.
// A portion's first token finds the token before it in before_state[slot], where the same workgroup, the only one that
// looks at that place in this step, then leaves the portion's last token.  One workgroup a token.
template <typename T>
__global__ void __launch_bounds__(256)
summed_embedding_kernel(const T* __restrict__ table, int64_t table_rows, const T* __restrict__ bigram, int64_t buckets, int64_t mul_prev,
                        int64_t mul_cur, const T* __restrict__ pos_table, int64_t pos_rows, const int32_t* __restrict__ ids,
                        const int32_t* __restrict__ positions, const int32_t* __restrict__ token_seq,
                        const int32_t* __restrict__ cu_seqlens_q, const int32_t* __restrict__ seq_starts,
                        const int32_t* __restrict__ state_slots, int32_t* before_state, float* __restrict__ out, int width,
                        int vec, int32_t* error_flag) {
    const int64_t t = blockIdx.x;
    const int id = ids[t], p = positions[t];
    const bool ok = id >= 0 && id < table_rows && (!pos_table || (p >= 0 && p < pos_rows));
    if (!ok && threadIdx.x == 0 && error_flag) atomicOr(error_flag, 1);
    const T* brow = nullptr;
    if (bigram) {
        const int s = token_seq[t];
        const int64_t first = cu_seqlens_q[s], next = cu_seqlens_q[s + 1];
        const int start = seq_starts[s], slot = state_slots[s];
        int64_t row = buckets;
        if (t > first || start > 0) {
            const int64_t before = t > first ? ids[t - 1] : before_state[slot];
            row = (max(before, (int64_t)0) * mul_prev + (int64_t)max(id, 0) * mul_cur) % buckets;
        }
        if (t == first) {
            __syncthreads();                             // (every thread has read the token before)
            if (threadIdx.x == 0) before_state[slot] = ids[next - 1];
        }
        brow = bigram + row * width;
    }
    const T* erow = table + (int64_t)(ok ? id : 0) * width;
    const T* prow = pos_table ? pos_table + (int64_t)(ok ? p : 0) * width : nullptr;
    if (vec) {
        for (int i = 8 * threadIdx.x; i < width; i += 8 * blockDim.x) {
            float v[8], b[8], q[8];
            load8(erow + i, v);
            if (brow) load8(brow + i, b);
            if (prow) load8(prow + i, q);
#pragma unroll
            for (int e = 0; e < 8; ++e) {
                if (brow) v[e] += b[e];
                if (prow) v[e] += q[e];
                if (!ok) v[e] = 0.f;
            }
            store8(out + t * width + i, v);
        }
        return;
    }
    for (int i = threadIdx.x; i < width; i += blockDim.x) {
        float v = to_float(erow[i]);
        if (brow) v += to_float(brow[i]);
        if (prow) v += to_float(prow[i]);
        out[t * width + i] = ok ? v : 0.f;
    }
}

NVA_EXPORT int NVA_NAME(nva_summed_embedding)(const void* table, int64_t table_rows, const void* bigram, int64_t buckets,
                                              int64_t mul_prev, int64_t mul_cur, const void* pos_table, int64_t pos_rows,
                                              const int32_t* ids, const int32_t* positions, const int32_t* token_seq,
                                              const int32_t* cu_seqlens_q, const int32_t* seq_starts, const int32_t* state_slots,
                                              int32_t* before_state, float* out, int64_t tokens, int width, int32_t* error_flag,
                                              hipStream_t stream) {
    if (tokens == 0) return 0;
    if (tokens < 0 || tokens > 0x7fffffff || width <= 0 || table_rows <= 0 || !table || !ids || !out || !positions)
        return nva_fail("summed_embedding: bad shape tokens=%lld width=%d rows=%lld", (long long)tokens, width, (long long)table_rows);
    if (bigram && (buckets <= 0 || mul_prev < 0 || mul_cur < 0 || mul_prev > 0x7fffffff || mul_cur > 0x7fffffff || !token_seq ||
                   !cu_seqlens_q || !seq_starts || !state_slots || !before_state))
        return nva_fail("summed_embedding: a bigram table needs its constants, the step's requests and their state");
    if (pos_table && pos_rows <= 0) return nva_fail("summed_embedding: an empty table of positions");
    const int threads = width >= 1024 ? 256 : (width >= 256 ? 128 : 64);
    const size_t vb = 8 * sizeof(elem_t);
    const int vec = width % 8 == 0 && nva_aligned(table, vb) && (!bigram || nva_aligned(bigram, vb)) &&
                    (!pos_table || nva_aligned(pos_table, vb)) && nva_aligned(out, 32);
    hipLaunchKernelGGL(summed_embedding_kernel<elem_t>, dim3((unsigned)tokens), dim3(threads), 0, stream, (const elem_t*)table,
                       table_rows, (const elem_t*)bigram, buckets, mul_prev, mul_cur, (const elem_t*)pos_table, pos_rows, ids,
                       positions, token_seq, cu_seqlens_q, seq_starts, state_slots, before_state, out, width, vec, error_flag);
    return nva_check_launch("summed_embedding");
}

// out[r] = x[r] over a float tensor of contiguous rows: a second copy of a stream that is updated in place.
__global__ void __launch_bounds__(256) copy_rows_kernel(const float* __restrict__ x, float* __restrict__ out, int64_t total) {
    for (int64_t i = (int64_t)blockIdx.x * blockDim.x + threadIdx.x; i < total; i += (int64_t)gridDim.x * blockDim.x) out[i] = x[i];
}
NVA_EXPORT int NVA_NAME(nva_copy_rows)(const float* x, float* out, int64_t total, hipStream_t stream) {
    if (total == 0) return 0;
    if (total < 0 || !x || !out) return nva_fail("copy_rows: bad arguments");
    const int64_t blocks = (total + 255) / 256;
    hipLaunchKernelGGL(copy_rows_kernel, dim3((unsigned)(blocks < 65536 ? blocks : 65536)), dim3(256), 0, stream, x, out, total);
    return nva_check_launch("copy_rows");
}

// out[t] = float(table[ids[t]]) * factor: the start of a residual stream kept in float (an embedding with a
// scale).  An id outside the table sets bit 0 of the flag and gives zeros.
template <typename T>
__global__ void __launch_bounds__(256)
gather_scale_rows_kernel(const T* __restrict__ table, int64_t table_stride, int64_t table_rows, const int32_t* __restrict__ ids,
                         float* __restrict__ out, int64_t out_stride, int width, float factor, int32_t* error_flag) {
    const int64_t t = blockIdx.x;
    const int id = ids[t];
    const bool ok = id >= 0 && id < table_rows;
    if (!ok && threadIdx.x == 0 && error_flag) atomicOr(error_flag, 1);
    const T* src = table + (int64_t)(ok ? id : 0) * table_stride;
    for (int i = threadIdx.x; i < width; i += blockDim.x) out[t * out_stride + i] = ok ? to_float(src[i]) * factor : 0.f;
}

NVA_EXPORT int NVA_NAME(nva_gather_scale_rows)(const void* table, int64_t table_stride, int64_t table_rows, const int32_t* ids,
                                               float* out, int64_t out_stride, int64_t count, int width, float factor,
                                               int32_t* error_flag, hipStream_t stream) {
    if (count == 0) return 0;
    if (count < 0 || count > 0x7fffffff || width <= 0 || table_rows <= 0 || !table || !ids || !out || out_stride < width)
        return nva_fail("gather_scale_rows: bad shape count=%lld width=%d rows=%lld", (long long)count, width,
                        (long long)table_rows);
    const int threads = width >= 1024 ? 256 : (width >= 256 ? 128 : 64);
    hipLaunchKernelGGL(gather_scale_rows_kernel<elem_t>, dim3((unsigned)count), dim3(threads), 0, stream,
                       (const elem_t*)table, table_stride, table_rows, ids, out, out_stride, width, factor, error_flag);
    return nva_check_launch("gather_scale_rows");
}

NVA_DEFINE_LAST_ERROR(nva_embed)
