// Element-wise steps behind matrix products:
//   clamped_gate   out = g sigmoid(alpha (g + cubic g^3)) (u + shift) of a (gate | up) projection, g capped and u clamped
//                  (the tanh form of gelu(g) u is alpha = 2 sqrt(2 / pi), cubic = 0.044715, shift = 0: (1 + tanh y) / 2 = sigmoid(2 y))
//   squared_relu   out = max(x, 0)^2
//   soft_cap       x = cap tanh(x / cap), in place
// Tensors are bf16 or fp32, arithmetic fp32.  V elements per thread: 8, or 1 where sizes or addresses do not allow it.
#include "nva_elem.h"

namespace nva {

template <typename T, int V>
__global__ __launch_bounds__(256) void clamped_gate_kernel(const T *__restrict__ x, int64_t stride, T *__restrict__ out,
                                                           int64_t total, int32_t per_row, int32_t inter, float limit,
                                                           float alpha, float cubic, float shift) {
    const int64_t idx = static_cast<int64_t>(blockIdx.x) * 256 + threadIdx.x;
    if (idx >= total) return;
    const int64_t row = idx / per_row;
    const int e = static_cast<int>(idx % per_row) * V;
    float g[V], u[V], y[V];
    load_f32<T, V>(x + row * stride + e, g);
    load_f32<T, V>(x + row * stride + inter + e, u);
#pragma unroll
    for (int i = 0; i < V; ++i) {
        const float gc = fminf(g[i], limit);
        const float uc = fminf(fmaxf(u[i], -limit), limit);
        y[i] = gc * sigmoid_of<T>(alpha * fmaf(cubic * gc, gc * gc, gc)) * (uc + shift);
    }
    store_f32<T, V>(out + row * inter + e, y);
}

template <typename T> struct SquaredRelu {
    static __device__ __forceinline__ float of(float v, float) {
        v = fmaxf(v, 0.f);
        return v * v;
    }
};
template <typename T> struct SoftCap {
    static __device__ __forceinline__ float of(float v, float cap) { return cap * tanh_of<T>(v / cap); }
};

// x and out may be the same
template <typename T, int V, typename F>
__global__ __launch_bounds__(256) void unary_kernel(const T *x, int64_t stride, T *out, int64_t total, int32_t per_row,
                                                    int32_t width, float p) {
    const int64_t idx = static_cast<int64_t>(blockIdx.x) * 256 + threadIdx.x;
    if (idx >= total) return;
    const int64_t row = idx / per_row;
    const int e = static_cast<int>(idx % per_row) * V;
    float v[V];
    load_f32<T, V>(x + row * stride + e, v);
#pragma unroll
    for (int i = 0; i < V; ++i) v[i] = F::of(v[i], p);
    store_f32<T, V>(out + row * width + e, v);
}

template <typename T, typename F>
static int launch_unary(const void *x, int64_t stride, void *out, int32_t rows, int32_t width, float p, hipStream_t s) {
    const bool vector = width % 8 == 0 && stride % 8 == 0 && aligned16(x) && aligned16(out);
    const int32_t per_row = vector ? width / 8 : width;
    const int64_t total = static_cast<int64_t>(rows) * per_row;
    if ((total + 255) / 256 > 0x7fffffffLL) return NVA_ERR_BAD_SHAPE;
    const dim3 grid(static_cast<uint32_t>((total + 255) / 256)), block(256);
    const T *xp = static_cast<const T *>(x);
    T *op = static_cast<T *>(out);
    if (vector) hipLaunchKernelGGL((unary_kernel<T, 8, F>), grid, block, 0, s, xp, stride, op, total, per_row, width, p);
    else hipLaunchKernelGGL((unary_kernel<T, 1, F>), grid, block, 0, s, xp, stride, op, total, per_row, width, p);
    return launch_status();
}

}  // namespace nva

extern "C" int nva_clamped_gate(const void *x, int64_t x_row_stride, void *out, int32_t rows, int32_t inter, float limit,
                                float alpha, float cubic, float shift, int32_t dtype, void *stream) {
    using namespace nva;
    if (rows < 0 || inter <= 0) return NVA_ERR_BAD_SHAPE;
    if (!known_dtype(dtype)) return NVA_ERR_UNSUPPORTED_GEOMETRY;
    if (rows == 0) return NVA_OK;
    if (!x || !out) return NVA_ERR_NULL_POINTER;
    if (x_row_stride < 2 * static_cast<int64_t>(inter)) return NVA_ERR_BAD_STRIDE;
    const bool vector = inter % 8 == 0 && x_row_stride % 8 == 0 && aligned16(x) && aligned16(out);
    const int32_t per_row = vector ? inter / 8 : inter;
    const int64_t total = static_cast<int64_t>(rows) * per_row;
    if ((total + 255) / 256 > 0x7fffffffLL) return NVA_ERR_BAD_SHAPE;
    const dim3 grid(static_cast<uint32_t>((total + 255) / 256)), block(256);
    hipStream_t s = static_cast<hipStream_t>(stream);
    if (dtype == NVA_DTYPE_BF16) {
        const bf16_t *xp = static_cast<const bf16_t *>(x);
        bf16_t *op = static_cast<bf16_t *>(out);
        if (vector) hipLaunchKernelGGL((clamped_gate_kernel<bf16_t, 8>), grid, block, 0, s, xp, x_row_stride, op, total, per_row, inter, limit, alpha, cubic, shift);
        else hipLaunchKernelGGL((clamped_gate_kernel<bf16_t, 1>), grid, block, 0, s, xp, x_row_stride, op, total, per_row, inter, limit, alpha, cubic, shift);
    } else {
        const float *xp = static_cast<const float *>(x);
        float *op = static_cast<float *>(out);
        if (vector) hipLaunchKernelGGL((clamped_gate_kernel<float, 8>), grid, block, 0, s, xp, x_row_stride, op, total, per_row, inter, limit, alpha, cubic, shift);
        else hipLaunchKernelGGL((clamped_gate_kernel<float, 1>), grid, block, 0, s, xp, x_row_stride, op, total, per_row, inter, limit, alpha, cubic, shift);
    }
    return launch_status();
}

extern "C" int nva_squared_relu(const void *x, int64_t x_row_stride, void *out, int32_t rows, int32_t width, int32_t dtype, void *stream) {
    using namespace nva;
    if (rows < 0 || width <= 0) return NVA_ERR_BAD_SHAPE;
    if (!known_dtype(dtype)) return NVA_ERR_UNSUPPORTED_GEOMETRY;
    if (rows == 0) return NVA_OK;
    if (!x || !out) return NVA_ERR_NULL_POINTER;
    if (x_row_stride < width || (x == out && x_row_stride != width)) return NVA_ERR_BAD_STRIDE;
    hipStream_t s = static_cast<hipStream_t>(stream);
    return dtype == NVA_DTYPE_BF16 ? launch_unary<bf16_t, SquaredRelu<bf16_t>>(x, x_row_stride, out, rows, width, 0.f, s)
                                   : launch_unary<float, SquaredRelu<float>>(x, x_row_stride, out, rows, width, 0.f, s);
}

extern "C" int nva_soft_cap(void *x, int32_t rows, int32_t width, float cap, int32_t dtype, void *stream) {
    using namespace nva;
    if (rows < 0 || width <= 0 || !(cap > 0.f)) return NVA_ERR_BAD_SHAPE;
    if (!known_dtype(dtype)) return NVA_ERR_UNSUPPORTED_GEOMETRY;
    if (rows == 0) return NVA_OK;
    if (!x) return NVA_ERR_NULL_POINTER;
    hipStream_t s = static_cast<hipStream_t>(stream);
    return dtype == NVA_DTYPE_BF16 ? launch_unary<bf16_t, SoftCap<bf16_t>>(x, width, x, rows, width, cap, s)
                                   : launch_unary<float, SoftCap<float>>(x, width, x, rows, width, cap, s);
}
