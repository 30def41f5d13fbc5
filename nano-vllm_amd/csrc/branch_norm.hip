// The residual step of layers whose mixer and feed-forward branch off the same point of the stream:
//   embed_norms     residual = embed[id] * scale, then the norms below
//   branches_norms  residual += mult * (gain1 * y1 + gain2 * sum_k weight_k y2_k)   (y2: the outputs of a
//                   row's experts, or one dense branch), then
//                   out1 = residual / rms * (offset + w1)     out2 = residual / rms * (offset + w2)
//   gated_norms     residual += sigmoid(z1 + b1) * y1 + sigmoid(z2 + b2) * sum_k weight_k y2_k   (z: gates of every element), then the
//                   norm, or the stream itself rounded
//   entry_norm      residual = y + step (y: a product in fp32), then the norm
// and of layers that norm what a sublayer gives instead of what it reads:
//   post_norms      y = weight * y1 + sum_k weight_k y2_k;  residual += y / rms * (offset + post), then
//                   out1 = residual, rounded, or its norm as above
// in one pass over the row.  Tensors are bf16 or fp32, the stream and all sums fp32.
#include "nva_elem.h"

#include <math.h>

namespace nva {

struct BranchArgs {
    const int64_t *ids;              // embed: token ids [rows]
    const void *x;                   // embed: table [vocab, width]; otherwise y1 [*, width] (may be null)
    int64_t x_stride;
    const void *gain1;               // [width] or null (1)
    const float *y1_weight;          // [*] one per row, or null (1)
    const void *y2;                  // [* x terms, width]: rows r * terms + k belong to row r (null: none)
    const float *term_weight;        // [*, terms] or null (1)
    int64_t weight_stride;           // between rows of y1_weight and term_weight
    const void *gain2;               // [width] or null (1)
    const void *gate;                // gated_norms: [*, width or 2 width] logits of the branches' gates
    const void *gate_bias;           // as many
    int64_t gate_stride;
    const float *product;            // entry_norm: [*, width] dense
    const void *step;                // entry_norm: [width]
    float *residual;                 // fp32 [*, width] dense
    const void *post;                // [width]: norm of the sum of the branches (post_norms)
    const void *w1, *w2;             // [width]; w2 null: one norm only; w1 null: out1 is the stream itself
    void *out1, *out2;               // [rows, width] dense (out1: row stride in elements)
    int64_t out1_stride;
    void *copy;                      // embed, optional: [rows, width], the stream itself, rounded
    int64_t copy_stride;
    const int32_t *rows_of;          // optional: output row r is computed from row rows_of[r], residual left alone
    int32_t *clear;                  // optional: counters set to zero
    int32_t clear_count, terms;
    int32_t rows, src_rows, width, vocab;
    float scale, mult, offset, eps;
};

__device__ __forceinline__ void clear_counters(const BranchArgs &a) {
    if (a.clear != nullptr && blockIdx.x == 0)
        for (int i = threadIdx.x; i < a.clear_count; i += 256) a.clear[i] = 0;
}

__device__ __forceinline__ int64_t branch_source_row(const BranchArgs &a, int row, bool embed) {
    if (embed || a.rows_of == nullptr) return row;
    return min(max(a.rows_of[row], 0), a.src_rows - 1);      // device data the host could not check
}

// v *= sigmoid(z + b)
template <typename T, int V>
__device__ __forceinline__ void channel_gate(const T *z, const T *b, float (&v)[V]) {
    float zs[V], bs[V];
    load_f32<T, V>(z, zs);
    load_f32<T, V>(b, bs);
#pragma unroll
    for (int i = 0; i < V; ++i) v[i] *= sigmoid_of<T>(zs[i] + bs[i]);
}

// V consecutive elements of the branches' sum
template <typename T, int V>
__device__ __forceinline__ void branch_sum(const BranchArgs &a, const T *xp, int64_t src, int e, float (&sum)[V]) {
    float v[V];
#pragma unroll
    for (int i = 0; i < V; ++i) sum[i] = 0.f;
    if (a.x != nullptr) {
        load_f32<T, V>(xp + e, v);
        if (a.gain1 != nullptr) load_f32<T, V>(static_cast<const T *>(a.gain1) + e, sum);
        if (a.y1_weight != nullptr) {
            const float w = a.y1_weight[src * a.weight_stride];
#pragma unroll
            for (int i = 0; i < V; ++i) v[i] *= w;
        }
        if (a.gate != nullptr) channel_gate<T, V>(static_cast<const T *>(a.gate) + src * a.gate_stride + e, static_cast<const T *>(a.gate_bias) + e, v);
#pragma unroll
        for (int i = 0; i < V; ++i) sum[i] = a.gain1 != nullptr ? sum[i] * v[i] : v[i];
    }
    if (a.y2 != nullptr) {
        float part[V];
#pragma unroll
        for (int i = 0; i < V; ++i) part[i] = 0.f;
        const T *yp = static_cast<const T *>(a.y2) + src * a.terms * a.width + e;
        const float *tw = a.term_weight != nullptr ? a.term_weight + src * a.weight_stride : nullptr;
        int k = 0;
        for (; k + 4 <= a.terms; k += 4) {
            float y[4][V], w[4];
#pragma unroll
            for (int j = 0; j < 4; ++j) {
                load_f32<T, V>(yp + static_cast<int64_t>(k + j) * a.width, y[j]);
                w[j] = tw != nullptr ? tw[k + j] : 1.0f;
            }
#pragma unroll
            for (int j = 0; j < 4; ++j)
#pragma unroll
                for (int i = 0; i < V; ++i) part[i] = fmaf(w[j], y[j][i], part[i]);
        }
        for (; k < a.terms; ++k) {
            const float w = tw != nullptr ? tw[k] : 1.0f;
            load_f32<T, V>(yp + static_cast<int64_t>(k) * a.width, v);
#pragma unroll
            for (int i = 0; i < V; ++i) part[i] = fmaf(w, v[i], part[i]);
        }
        if (a.gate != nullptr)
            channel_gate<T, V>(static_cast<const T *>(a.gate) + src * a.gate_stride + a.width + e, static_cast<const T *>(a.gate_bias) + a.width + e, part);
        float gain[V];
        if (a.gain2 != nullptr) load_f32<T, V>(static_cast<const T *>(a.gain2) + e, gain);
#pragma unroll
        for (int i = 0; i < V; ++i) sum[i] = a.gain2 != nullptr ? fmaf(gain[i], part[i], sum[i]) : sum[i] + part[i];
    }
}

enum Step { kEmbed, kBranches, kPostNorm, kEntry };

// V consecutive elements of the new residual; rstd: of the branches' sum (kPostNorm)
template <typename T, int V, Step kStep>
__device__ __forceinline__ void new_residual(const BranchArgs &a, const T *xp, int64_t src, int e, float rstd, float (&r)[V]) {
    float v[V];
    if (kStep == kEmbed) {
        load_f32<T, V>(xp + e, v);
#pragma unroll
        for (int i = 0; i < V; ++i) r[i] = v[i] * a.scale;
        return;
    }
    if (kStep == kEntry) {
        load_f32<float, V>(a.product + src * a.width + e, r);
        load_f32<T, V>(static_cast<const T *>(a.step) + e, v);
#pragma unroll
        for (int i = 0; i < V; ++i) r[i] += v[i];
        return;
    }
    load_f32<float, V>(a.residual + src * a.width + e, r);
    branch_sum<T, V>(a, xp, src, e, v);
    if (kStep == kPostNorm) {
        float w[V];
        load_f32<T, V>(static_cast<const T *>(a.post) + e, w);
#pragma unroll
        for (int i = 0; i < V; ++i) r[i] = fmaf(v[i] * rstd, a.offset + w[i], r[i]);
    } else {
#pragma unroll
        for (int i = 0; i < V; ++i) r[i] = fmaf(a.mult, v[i], r[i]);
    }
}

// The row in registers, 8 elements per access (width % 8 == 0, width <= 4096): WPR = 1, one wavefront per row, NC pieces of
// 512 elements; WPR = 4 (few rows), a workgroup per row, NC pieces of 2048.
template <typename T, int NC, int WPR, Step kStep>
__global__ __launch_bounds__(256) void branch_norm_kernel(BranchArgs a) {
    __shared__ float sh[2][4];
    clear_counters(a);
    constexpr int kPiece = 512 * WPR;
    const int at0 = (threadIdx.x & (64 * WPR - 1)) * 8;
    const int row = WPR == 1 ? blockIdx.x * 4 + (threadIdx.x >> 6) : blockIdx.x;
    if (row >= a.rows) return;
    const int64_t src = branch_source_row(a, row, kStep == kEmbed);
    int64_t xrow = src;
    if (kStep == kEmbed) xrow = min(max(a.ids[row], static_cast<int64_t>(0)), static_cast<int64_t>(a.vocab) - 1);
    const T *xp = static_cast<const T *>(a.x) + xrow * a.x_stride;
    auto rstd_of = [&](float sq, int which) __attribute__((always_inline)) -> float {
        sq = wave_sum(sq);
        if (WPR > 1) {
            if ((threadIdx.x & 63) == 0) sh[which][threadIdx.x >> 6] = sq;
            __syncthreads();
            sq = (sh[which][0] + sh[which][1]) + (sh[which][2] + sh[which][3]);
        }
        return rsqrtf(sq / static_cast<float>(a.width) + a.eps);
    };
    float r[NC][8];
    float sq = 0.f;
    if constexpr (kStep == kPostNorm) {
        float y[NC][8];
#pragma unroll
        for (int c = 0; c < NC; ++c) {
            const int e = c * kPiece + at0;
            if (e < a.width) {
                load_f32<float, 8>(a.residual + src * a.width + e, r[c]);
                branch_sum<T, 8>(a, xp, src, e, y[c]);
#pragma unroll
                for (int i = 0; i < 8; ++i) sq = fmaf(y[c][i], y[c][i], sq);
            }
        }
        const float rstd = rstd_of(sq, 0);
        sq = 0.f;
#pragma unroll
        for (int c = 0; c < NC; ++c) {
            const int e = c * kPiece + at0;
            if (e < a.width) {
                float w[8];
                load_f32<T, 8>(static_cast<const T *>(a.post) + e, w);
#pragma unroll
                for (int i = 0; i < 8; ++i) {
                    r[c][i] = fmaf(y[c][i] * rstd, a.offset + w[i], r[c][i]);
                    sq = fmaf(r[c][i], r[c][i], sq);
                }
                if (a.rows_of == nullptr) store_f32<float, 8>(a.residual + src * a.width + e, r[c]);
            }
        }
    } else {
#pragma unroll
        for (int c = 0; c < NC; ++c) {
            const int e = c * kPiece + at0;
            if (e < a.width) {
                new_residual<T, 8, kStep>(a, xp, src, e, 0.f, r[c]);
                if (kStep == kEmbed || a.rows_of == nullptr) store_f32<float, 8>(a.residual + src * a.width + e, r[c]);
                if (kStep == kEmbed && a.copy != nullptr) store_f32<T, 8>(static_cast<T *>(a.copy) + row * a.copy_stride + e, r[c]);
#pragma unroll
                for (int i = 0; i < 8; ++i) sq = fmaf(r[c][i], r[c][i], sq);
            }
        }
    }
    const int64_t at = static_cast<int64_t>(row) * a.width, at1 = row * a.out1_stride;
    if (a.w1 == nullptr) {                                   // (the same for every row)
#pragma unroll
        for (int c = 0; c < NC; ++c) {
            const int e = c * kPiece + at0;
            if (e < a.width) store_f32<T, 8>(static_cast<T *>(a.out1) + at1 + e, r[c]);
        }
        return;
    }
    const float rstd = rstd_of(sq, 1);
#pragma unroll
    for (int c = 0; c < NC; ++c) {
        const int e = c * kPiece + at0;
        if (e < a.width) {
            float w[8], y[8];
            load_f32<T, 8>(static_cast<const T *>(a.w1) + e, w);
#pragma unroll
            for (int i = 0; i < 8; ++i) y[i] = r[c][i] * rstd * (a.offset + w[i]);
            store_f32<T, 8>(static_cast<T *>(a.out1) + at1 + e, y);
            if (a.w2 != nullptr) {
                load_f32<T, 8>(static_cast<const T *>(a.w2) + e, w);
#pragma unroll
                for (int i = 0; i < 8; ++i) y[i] = r[c][i] * rstd * (a.offset + w[i]);
                store_f32<T, 8>(static_cast<T *>(a.out2) + at + e, y);
            }
        }
    }
}

// Any width: one workgroup per row; a thread re-reads the residual elements it wrote itself (or, where
// they are not written, computes them again).
template <typename T, Step kStep>
__global__ __launch_bounds__(256) void branch_norm_any_kernel(BranchArgs a) {
    __shared__ float sh[2][4];
    clear_counters(a);
    const int row = blockIdx.x;
    const int64_t src = branch_source_row(a, row, kStep == kEmbed);
    int64_t xrow = src;
    if (kStep == kEmbed) xrow = min(max(a.ids[row], static_cast<int64_t>(0)), static_cast<int64_t>(a.vocab) - 1);
    const T *xp = static_cast<const T *>(a.x) + xrow * a.x_stride;
    const bool keep = kStep == kEmbed || a.rows_of == nullptr;
    auto rstd_of = [&](float sq, int which) -> float {
        sq = wave_sum(sq);
        if ((threadIdx.x & 63) == 0) sh[which][threadIdx.x >> 6] = sq;
        __syncthreads();
        return rsqrtf(((sh[which][0] + sh[which][1]) + (sh[which][2] + sh[which][3])) / static_cast<float>(a.width) + a.eps);
    };
    float sq = 0.f, post_rstd = 0.f;
    if (kStep == kPostNorm) {
        for (int e = threadIdx.x; e < a.width; e += 256) {
            float y[1];
            branch_sum<T, 1>(a, xp, src, e, y);
            sq = fmaf(y[0], y[0], sq);
        }
        post_rstd = rstd_of(sq, 0);
        sq = 0.f;
    }
    for (int e = threadIdx.x; e < a.width; e += 256) {
        float r[1];
        new_residual<T, 1, kStep>(a, xp, src, e, post_rstd, r);
        if (keep) a.residual[src * a.width + e] = r[0];
        if (kStep == kEmbed && a.copy != nullptr) static_cast<T *>(a.copy)[row * a.copy_stride + e] = Elem<T>::from_f32(r[0]);
        sq = fmaf(r[0], r[0], sq);
    }
    const float rstd = rstd_of(sq, 1);
    const int64_t at = static_cast<int64_t>(row) * a.width, at1 = row * a.out1_stride;
    for (int e = threadIdx.x; e < a.width; e += 256) {
        float r[1];
        if (keep) r[0] = a.residual[src * a.width + e];
        else new_residual<T, 1, kStep>(a, xp, src, e, post_rstd, r);
        const float y = a.w1 == nullptr ? r[0] : r[0] * rstd * (a.offset + Elem<T>::to_f32(static_cast<const T *>(a.w1)[e]));
        static_cast<T *>(a.out1)[at1 + e] = Elem<T>::from_f32(y);
        if (a.w2 != nullptr)
            static_cast<T *>(a.out2)[at + e] = Elem<T>::from_f32(r[0] * rstd * (a.offset + Elem<T>::to_f32(static_cast<const T *>(a.w2)[e])));
    }
}

template <typename T, Step kStep>
static int launch_branch_norm(const BranchArgs &a, hipStream_t s) {
    const bool vector = a.width % 8 == 0 && a.width <= 4096 && a.x_stride % 8 == 0 && aligned16(a.x) && aligned16(a.residual) &&
                        aligned16(a.gain1) && aligned16(a.y2) && aligned16(a.gain2) && aligned16(a.post) && aligned16(a.w1) && aligned16(a.w2) &&
                        aligned16(a.out1) && aligned16(a.out2) && a.out1_stride % 8 == 0 && a.copy_stride % 8 == 0 && aligned16(a.copy) &&
                        a.gate_stride % 8 == 0 && aligned16(a.gate) && aligned16(a.gate_bias) && aligned16(a.product) && aligned16(a.step);
    if (!vector) {
        hipLaunchKernelGGL((branch_norm_any_kernel<T, kStep>), dim3(a.rows), dim3(256), 0, s, a);
        return launch_status();
    }
    const dim3 block(256);
    if (a.rows <= 1024) {
        if (a.width <= 2048) hipLaunchKernelGGL((branch_norm_kernel<T, 1, 4, kStep>), dim3(a.rows), block, 0, s, a);
        else hipLaunchKernelGGL((branch_norm_kernel<T, 2, 4, kStep>), dim3(a.rows), block, 0, s, a);
        return launch_status();
    }
    const dim3 grid((a.rows + 3) / 4);
    switch ((a.width + 511) / 512) {
        case 1: hipLaunchKernelGGL((branch_norm_kernel<T, 1, 1, kStep>), grid, block, 0, s, a); break;
        case 2: hipLaunchKernelGGL((branch_norm_kernel<T, 2, 1, kStep>), grid, block, 0, s, a); break;
        case 3: case 4: hipLaunchKernelGGL((branch_norm_kernel<T, 4, 1, kStep>), grid, block, 0, s, a); break;
        default: hipLaunchKernelGGL((branch_norm_kernel<T, 8, 1, kStep>), grid, block, 0, s, a); break;
    }
    return launch_status();
}

}  // namespace nva

extern "C" int nva_embed_rms_norms(const int64_t *ids, const void *table, float scale, const void *weight1, const void *weight2,
                                   float weight_offset, float *residual, void *out1, int64_t out1_row_stride, void *out2, void *copy, int64_t copy_row_stride,
                                   int32_t *clear, int32_t clear_count, int32_t rows, int32_t width, int32_t vocab, float eps, int32_t dtype,
                                   void *stream) {
    using namespace nva;
    if (rows < 0 || width <= 0 || vocab <= 0 || clear_count < 0) return NVA_ERR_BAD_SHAPE;
    if (!known_dtype(dtype)) return NVA_ERR_UNSUPPORTED_GEOMETRY;
    if (rows == 0) return NVA_OK;
    if (!ids || !table || !residual || !out1 || (weight2 && (!weight1 || !out2))) return NVA_ERR_NULL_POINTER;
    if (out1_row_stride < width || (copy && copy_row_stride < width)) return NVA_ERR_BAD_STRIDE;
    BranchArgs a{};
    a.out1_stride = out1_row_stride; a.copy = copy; a.copy_stride = copy ? copy_row_stride : 0;
    a.ids = ids; a.x = table; a.x_stride = width; a.residual = residual; a.w1 = weight1; a.w2 = weight2; a.out1 = out1; a.out2 = out2;
    a.clear = clear; a.clear_count = clear ? clear_count : 0; a.rows = rows; a.src_rows = rows; a.width = width; a.vocab = vocab;
    a.scale = scale; a.offset = weight_offset; a.eps = eps;
    hipStream_t s = static_cast<hipStream_t>(stream);
    return dtype == NVA_DTYPE_BF16 ? launch_branch_norm<bf16_t, kEmbed>(a, s) : launch_branch_norm<float, kEmbed>(a, s);
}

extern "C" int nva_branches_rms_norms(const void *y1, int64_t y1_row_stride, const void *gain1, const void *y2,
                                      const float *term_weight, int32_t terms, const void *gain2, float mult, float *residual,
                                      const void *weight1, const void *weight2, float weight_offset, void *out1, void *out2,
                                      const int32_t *rows_of, int32_t *clear, int32_t clear_count, int32_t rows,
                                      int32_t src_rows, int32_t width, float eps, int32_t dtype, void *stream) {
    using namespace nva;
    if (rows < 0 || src_rows < 0 || width <= 0 || terms < 0 || clear_count < 0) return NVA_ERR_BAD_SHAPE;
    if (!known_dtype(dtype)) return NVA_ERR_UNSUPPORTED_GEOMETRY;
    if (rows == 0) return NVA_OK;
    if (src_rows == 0 || (!rows_of && rows != src_rows) || (y2 && terms == 0)) return NVA_ERR_BAD_SHAPE;
    if (!residual || !weight1 || !out1 || (weight2 && !out2)) return NVA_ERR_NULL_POINTER;
    if (y1 && y1_row_stride < width) return NVA_ERR_BAD_STRIDE;
    BranchArgs a{};
    a.x = y1; a.x_stride = y1 ? y1_row_stride : 0; a.gain1 = gain1; a.y2 = y2; a.term_weight = term_weight; a.weight_stride = terms; a.terms = terms; a.gain2 = gain2;
    a.mult = mult; a.residual = residual; a.w1 = weight1; a.w2 = weight2; a.offset = weight_offset; a.out1 = out1; a.out2 = out2;
    a.rows_of = rows_of; a.clear = clear; a.clear_count = clear ? clear_count : 0; a.rows = rows; a.src_rows = src_rows;
    a.out1_stride = width; a.width = width; a.eps = eps;
    hipStream_t s = static_cast<hipStream_t>(stream);
    return dtype == NVA_DTYPE_BF16 ? launch_branch_norm<bf16_t, kBranches>(a, s) : launch_branch_norm<float, kBranches>(a, s);
}

extern "C" int nva_post_rms_norms(const void *y1, int64_t y1_row_stride, const float *y1_weight, const void *y2,
                                  const float *term_weight, int64_t weight_row_stride, int32_t terms, const void *post_weight,
                                  float *residual, const void *next_weight, float weight_offset, void *out, const int32_t *rows_of,
                                  int32_t *clear, int32_t clear_count, int32_t rows, int32_t src_rows, int32_t width, float eps,
                                  int32_t dtype, void *stream) {
    using namespace nva;
    if (rows < 0 || src_rows < 0 || width <= 0 || terms < 0 || clear_count < 0) return NVA_ERR_BAD_SHAPE;
    if (!known_dtype(dtype)) return NVA_ERR_UNSUPPORTED_GEOMETRY;
    if (rows == 0) return NVA_OK;
    if (src_rows == 0 || (!rows_of && rows != src_rows) || (y2 && terms == 0)) return NVA_ERR_BAD_SHAPE;
    if (!residual || !post_weight || !out || (!y1 && !y2)) return NVA_ERR_NULL_POINTER;
    if ((y1 && y1_row_stride < width) || (y1_weight && weight_row_stride < 1) || (term_weight && weight_row_stride < terms)) return NVA_ERR_BAD_STRIDE;
    BranchArgs a{};
    a.x = y1; a.x_stride = y1 ? y1_row_stride : 0; a.y1_weight = y1_weight; a.y2 = y2; a.term_weight = term_weight; a.weight_stride = weight_row_stride;
    a.terms = terms; a.post = post_weight; a.residual = residual; a.w1 = next_weight; a.offset = weight_offset; a.out1 = out;
    a.rows_of = rows_of; a.clear = clear; a.clear_count = clear ? clear_count : 0; a.rows = rows; a.src_rows = src_rows;
    a.out1_stride = width; a.width = width; a.eps = eps;
    hipStream_t s = static_cast<hipStream_t>(stream);
    return dtype == NVA_DTYPE_BF16 ? launch_branch_norm<bf16_t, kPostNorm>(a, s) : launch_branch_norm<float, kPostNorm>(a, s);
}

extern "C" int nva_gated_rms_norm(const void *y1, int64_t y1_row_stride, const void *y2, int32_t terms, const void *gate,
                                  int64_t gate_row_stride, const void *gate_bias, float *residual, const void *weight, float weight_offset,
                                  void *out, int64_t out_row_stride, const int32_t *rows_of, int32_t *clear, int32_t clear_count,
                                  int32_t rows, int32_t src_rows, int32_t width, float eps, int32_t dtype, void *stream) {
    using namespace nva;
    if (rows < 0 || src_rows < 0 || width <= 0 || terms < 0 || clear_count < 0) return NVA_ERR_BAD_SHAPE;
    if (!known_dtype(dtype)) return NVA_ERR_UNSUPPORTED_GEOMETRY;
    if (rows == 0) return NVA_OK;
    if (src_rows == 0 || (!rows_of && rows != src_rows) || (y2 && terms == 0)) return NVA_ERR_BAD_SHAPE;
    if (!y1 || !gate || !gate_bias || !residual || !out) return NVA_ERR_NULL_POINTER;
    if (y1_row_stride < width || gate_row_stride < (y2 ? 2 : 1) * static_cast<int64_t>(width) || out_row_stride < width) return NVA_ERR_BAD_STRIDE;
    BranchArgs a{};
    a.x = y1; a.x_stride = y1_row_stride; a.y2 = y2; a.terms = terms; a.weight_stride = terms; a.gate = gate; a.gate_stride = gate_row_stride;
    a.gate_bias = gate_bias; a.mult = 1.0f; a.residual = residual; a.w1 = weight; a.offset = weight_offset; a.out1 = out; a.out1_stride = out_row_stride;
    a.rows_of = rows_of; a.clear = clear; a.clear_count = clear ? clear_count : 0; a.rows = rows; a.src_rows = src_rows;
    a.width = width; a.eps = eps;
    hipStream_t s = static_cast<hipStream_t>(stream);
    return dtype == NVA_DTYPE_BF16 ? launch_branch_norm<bf16_t, kBranches>(a, s) : launch_branch_norm<float, kBranches>(a, s);
}

extern "C" int nva_entry_rms_norm(const float *product, const void *step, float *residual, const void *weight, float weight_offset, void *out,
                                  int32_t *clear, int32_t clear_count, int32_t rows, int32_t width, float eps, int32_t dtype, void *stream) {
    using namespace nva;
    if (rows < 0 || width <= 0 || clear_count < 0) return NVA_ERR_BAD_SHAPE;
    if (!known_dtype(dtype)) return NVA_ERR_UNSUPPORTED_GEOMETRY;
    if (rows == 0) return NVA_OK;
    if (!product || !step || !residual || !weight || !out) return NVA_ERR_NULL_POINTER;
    BranchArgs a{};
    a.product = product; a.step = step; a.residual = residual; a.w1 = weight; a.offset = weight_offset; a.out1 = out; a.out1_stride = width;
    a.clear = clear; a.clear_count = clear ? clear_count : 0; a.rows = rows; a.src_rows = rows; a.width = width; a.eps = eps;
    hipStream_t s = static_cast<hipStream_t>(stream);
    return dtype == NVA_DTYPE_BF16 ? launch_branch_norm<bf16_t, kEntry>(a, s) : launch_branch_norm<float, kEntry>(a, s);
}
