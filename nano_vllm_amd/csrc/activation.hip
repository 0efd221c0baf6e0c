// Gating of a feed-forward: out[t, i] = act(x[t, i]) * x[t, inner + i].  SwiGLU is act = silu,
// silu(g) = g * sigmoid(g) (nanovllm/layers/activation.py:8-11); the other activations are relu and
// the tanh form of gelu, 0.5 g (1 + tanh(sqrt(2/pi) (g + 0.044715 g^3))).  Computed in float and
// rounded once.
#include "common.h"

#define NVA_ACT_SILU 0
#define NVA_ACT_RELU 1
#define NVA_ACT_GELU_TANH 2

template <int ACT> __device__ __forceinline__ float nva_act(float g) {
    if (ACT == NVA_ACT_RELU) return fmaxf(g, 0.f);
    if (ACT == NVA_ACT_GELU_TANH) return 0.5f * g * (1.f + tanhf(0.7978845608028654f * (g + 0.044715f * g * g * g)));
    return g / (1.f + nva_exp(-g));
}

template <typename T, bool VEC, int ACT>
__global__ void __launch_bounds__(256)
act_mul_kernel(const T* __restrict__ x, int64_t x_stride, T* __restrict__ out, int64_t out_stride, int inner) {
    const int64_t row = blockIdx.y;
    const T* gate = x + row * x_stride;
    const T* up = gate + inner;
    T* o = out + row * out_stride;
    if (VEC) {
        const int i = (blockIdx.x * blockDim.x + threadIdx.x) * 8;
        if (i >= inner) return;
        float g[8], u[8];
        load8(gate + i, g);
        load8(up + i, u);
#pragma unroll
        for (int j = 0; j < 8; ++j) g[j] = nva_act<ACT>(g[j]) * u[j];
        store8(o + i, g);
    } else {
        const int i = blockIdx.x * blockDim.x + threadIdx.x;
        if (i >= inner) return;
        const float g = to_float(gate[i]);
        o[i] = from_float<T>(nva_act<ACT>(g) * to_float(up[i]));
    }
}

template <int ACT>
static int launch_act_mul(const void* x, int64_t x_stride, void* out, int64_t out_stride, int64_t rows, int inner,
                          hipStream_t stream) {
    if (rows == 0) return 0;
    if (rows < 0 || rows > 65535LL * 65535LL || inner <= 0)
        return nva_fail("act_mul: bad shape rows=%lld inner=%d", (long long)rows, inner);
    const size_t vb = 8 * sizeof(elem_t);
    const bool vec = inner % 8 == 0 && x_stride % 8 == 0 && out_stride % 8 == 0 && nva_aligned(x, vb) &&
                     nva_aligned(out, vb);
    // grid.y is limited to 65535 rows per launch
    const elem_t* xp = (const elem_t*)x;
    elem_t* op = (elem_t*)out;
    for (int64_t r0 = 0; r0 < rows; r0 += 65535) {
        const unsigned nr = (unsigned)((rows - r0) < 65535 ? (rows - r0) : 65535);
        if (vec) {
            dim3 grid((inner / 8 + 255) / 256, nr);
            hipLaunchKernelGGL((act_mul_kernel<elem_t, true, ACT>), grid, dim3(256), 0, stream, xp + r0 * x_stride,
                               x_stride, op + r0 * out_stride, out_stride, inner);
        } else {
            dim3 grid((inner + 255) / 256, nr);
            hipLaunchKernelGGL((act_mul_kernel<elem_t, false, ACT>), grid, dim3(256), 0, stream, xp + r0 * x_stride,
                               x_stride, op + r0 * out_stride, out_stride, inner);
        }
    }
    return nva_check_launch("act_mul");
}

// act: 0 silu, 1 relu, 2 gelu (tanh form)
NVA_EXPORT int NVA_NAME(nva_act_mul)(const void* x, int64_t x_stride, void* out, int64_t out_stride,
                                     int64_t rows, int inner, int act, hipStream_t stream) {
    switch (act) {
        case NVA_ACT_SILU: return launch_act_mul<NVA_ACT_SILU>(x, x_stride, out, out_stride, rows, inner, stream);
        case NVA_ACT_RELU: return launch_act_mul<NVA_ACT_RELU>(x, x_stride, out, out_stride, rows, inner, stream);
        case NVA_ACT_GELU_TANH: return launch_act_mul<NVA_ACT_GELU_TANH>(x, x_stride, out, out_stride, rows, inner, stream);
    }
    return nva_fail("act_mul: unknown activation %d", act);
}

NVA_EXPORT int NVA_NAME(nva_silu_mul)(const void* x, int64_t x_stride, void* out, int64_t out_stride,
                                      int64_t rows, int inner, hipStream_t stream) {
    return launch_act_mul<NVA_ACT_SILU>(x, x_stride, out, out_stride, rows, inner, stream);
}

// An activation without a gate: out[t, i] = act(x[t, i]); act by the codes of nva_plain_act.
// Eight entries a thread where rows and pointers allow.
template <typename T>
__global__ void __launch_bounds__(256)
act8_kernel(const T* __restrict__ x, int64_t x_stride, T* __restrict__ out, int64_t out_stride, int64_t rows, int width8, int act) {
    const int64_t idx = (int64_t)blockIdx.x * blockDim.x + threadIdx.x;
    if (idx >= rows * width8) return;
    const int64_t r = idx / width8;
    const int i = (int)(idx % width8) * 8;
    float v[8];
    load8(x + r * x_stride + i, v);
#pragma unroll
    for (int e = 0; e < 8; ++e) v[e] = nva_plain_act(act, v[e]);
    store8(out + r * out_stride + i, v);
}

// The same from a product that was left as partial sums: out[t, i] = act(round(sum + bias)).
template <typename T>
__global__ void __launch_bounds__(256)
act_of_partials_kernel(PartialInput part, T* __restrict__ out, int64_t out_stride, int width, int act) {
    const int64_t r = blockIdx.y;
    const int i = blockIdx.x * blockDim.x + threadIdx.x;
    if (i >= width) return;
    out[r * out_stride + i] = from_float<T>(nva_plain_act(act, partial_value<T>(part, r, width, i)));
}

template <typename T>
__global__ void __launch_bounds__(256)
act_kernel(const T* __restrict__ x, int64_t x_stride, T* __restrict__ out, int64_t out_stride, int64_t rows, int width, int act) {
    const int64_t idx = (int64_t)blockIdx.x * blockDim.x + threadIdx.x;
    if (idx >= rows * width) return;
    const int64_t r = idx / width;
    const int i = (int)(idx % width);
    out[r * out_stride + i] = from_float<T>(nva_plain_act(act, to_float(x[r * x_stride + i])));
}

NVA_EXPORT int NVA_NAME(nva_act)(const void* x, int64_t x_stride, void* out, int64_t out_stride, int64_t rows, int width,
                                 int act, hipStream_t stream) {
    if (rows == 0) return 0;
    if (rows < 0 || width <= 0 || act < 0 || act > 4) return nva_fail("act: bad shape rows=%lld width=%d or activation %d", (long long)rows, width, act);
    const int64_t total = rows * width;
    if ((total + 255) / 256 > 0x7fffffff) return nva_fail("act: too many entries");
    const size_t vb = 8 * sizeof(elem_t);
    if (width % 8 == 0 && x_stride % 8 == 0 && out_stride % 8 == 0 && nva_aligned(x, vb) && nva_aligned(out, vb)) {
        hipLaunchKernelGGL((act8_kernel<elem_t>), dim3((unsigned)((total / 8 + 255) / 256)), dim3(256), 0, stream,
                           (const elem_t*)x, x_stride, (elem_t*)out, out_stride, rows, width / 8, act);
        return nva_check_launch("act");
    }
    hipLaunchKernelGGL((act_kernel<elem_t>), dim3((unsigned)((total + 255) / 256)), dim3(256), 0, stream, (const elem_t*)x,
                       x_stride, (elem_t*)out, out_stride, rows, width, act);
    return nva_check_launch("act");
}

// sums: float [splits][rows][width], with an optional bias of elements [width].
NVA_EXPORT int NVA_NAME(nva_act_of_partials)(const float* sums, int splits, int64_t split_stride, const void* bias, void* out,
                                             int64_t out_stride, int64_t rows, int width, int act, hipStream_t stream) {
    if (rows == 0) return 0;
    if (rows < 0 || rows > 65535 || width <= 0 || act < 0 || act > 4 || !sums || splits <= 0 || split_stride < rows * (int64_t)width ||
        !out || out_stride < width)
        return nva_fail("act_of_partials: bad shape rows=%lld width=%d splits=%d or activation %d", (long long)rows, width, splits, act);
    const PartialInput part{sums, splits, split_stride, bias};
    hipLaunchKernelGGL((act_of_partials_kernel<elem_t>), dim3((width + 255) / 256, (unsigned)rows), dim3(256), 0, stream, part,
                       (elem_t*)out, out_stride, width, act);
    return nva_check_launch("act_of_partials");
}

// The same times a row of a table: out[t, i] = act(x[t, i]) * table[ids[t], offset + i], in float, rounded once.  x comes as
// elements or as a product's partial sums.  An id outside the table sets bit 0 of the flag and gives zeros.
template <typename T>
__global__ void __launch_bounds__(256)
act_mul_rows_kernel(const T* __restrict__ x, int64_t x_stride, PartialInput part, const T* __restrict__ table, int64_t table_stride,
                    int64_t table_rows, int offset, const int32_t* __restrict__ ids, T* __restrict__ out, int64_t out_stride,
                    int64_t rows, int width, int act, int32_t* error_flag) {
    const int64_t idx = (int64_t)blockIdx.x * blockDim.x + threadIdx.x;
    if (idx >= rows * width) return;
    const int64_t r = idx / width;
    const int i = (int)(idx % width);
    const int id = ids[r];
    const bool ok = id >= 0 && id < table_rows;
    if (!ok && i == 0 && error_flag) atomicOr(error_flag, 1);
    const float e = ok ? to_float(table[(int64_t)id * table_stride + offset + i]) : 0.f;
    const float v = part.sums ? partial_value<T>(part, r, width, i) : to_float(x[r * x_stride + i]);
    out[r * out_stride + i] = from_float<T>(nva_plain_act(act, v) * e);
}

// x: elements [rows, width], or (sums) partial sums [splits][rows][width] with an optional bias.
NVA_EXPORT int NVA_NAME(nva_act_mul_rows)(const void* x, int64_t x_stride, const float* sums, int splits, int64_t split_stride,
                                          const void* bias, const void* table, int64_t table_stride, int64_t table_rows, int offset,
                                          const int32_t* ids, void* out, int64_t out_stride, int64_t rows, int width, int act,
                                          int32_t* error_flag, hipStream_t stream) {
    if (rows == 0) return 0;
    if (rows < 0 || width <= 0 || act < 0 || act > 4 || (!x && !sums) || !table || !ids || !out || table_rows <= 0 || offset < 0 ||
        table_stride < (int64_t)offset + width || out_stride < width)
        return nva_fail("act_mul_rows: bad shape rows=%lld width=%d offset=%d or activation %d", (long long)rows, width, offset, act);
    if (sums && (splits <= 0 || split_stride < rows * (int64_t)width)) return nva_fail("act_mul_rows: bad partial sums");
    const int64_t total = rows * width;
    if ((total + 255) / 256 > 0x7fffffff) return nva_fail("act_mul_rows: too many entries");
    const PartialInput part{sums, splits, split_stride, bias};
    hipLaunchKernelGGL((act_mul_rows_kernel<elem_t>), dim3((unsigned)((total + 255) / 256)), dim3(256), 0, stream, (const elem_t*)x,
                       x_stride, part, (const elem_t*)table, table_stride, table_rows, offset, ids, (elem_t*)out, out_stride, rows,
                       width, act, error_flag);
    return nva_check_launch("act_mul_rows");
}

// A gate on finished outputs: out[t, i] = x[t, i] * sigmoid(g[t, i]), in float, rounded once (out may be x).
template <typename T>
__global__ void __launch_bounds__(256)
sigmoid_mul_kernel(const T* __restrict__ x, int64_t x_stride, const T* __restrict__ g, int64_t g_stride, T* __restrict__ out,
                   int64_t out_stride, int64_t rows, int width) {
    const int64_t idx = (int64_t)blockIdx.x * blockDim.x + threadIdx.x;
    if (idx >= rows * width) return;
    const int64_t r = idx / width;
    const int i = (int)(idx % width);
    const float gate = 1.f / (1.f + nva_exp(-to_float(g[r * g_stride + i])));
    out[r * out_stride + i] = from_float<T>(to_float(x[r * x_stride + i]) * gate);
}

NVA_EXPORT int NVA_NAME(nva_sigmoid_mul)(const void* x, int64_t x_stride, const void* g, int64_t g_stride, void* out,
                                         int64_t out_stride, int64_t rows, int width, hipStream_t stream) {
    if (rows == 0) return 0;
    if (rows < 0 || width <= 0 || !x || !g || !out) return nva_fail("sigmoid_mul: bad shape rows=%lld width=%d", (long long)rows, width);
    const int64_t total = rows * width;
    if ((total + 255) / 256 > 0x7fffffff) return nva_fail("sigmoid_mul: too many entries");
    hipLaunchKernelGGL((sigmoid_mul_kernel<elem_t>), dim3((unsigned)((total + 255) / 256)), dim3(256), 0, stream,
                       (const elem_t*)x, x_stride, (const elem_t*)g, g_stride, (elem_t*)out, out_stride, rows, width);
    return nva_check_launch("sigmoid_mul");
}

NVA_DEFINE_LAST_ERROR(nva_activation)
