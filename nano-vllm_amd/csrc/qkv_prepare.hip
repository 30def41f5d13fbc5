// What an attention layer does with its projections before it attends: bias, norm of queries and keys (of every head by
// itself, or over all of a projection's rows at once; with a weight or without), norm of every head's values, rotation, queries out, keys and values into the paged cache.
// One pass over the row; tensors are bf16 or fp32, arithmetic fp32.
#include "nva_elem.h"

#include <math.h>

namespace nva {

struct QkvArgs {
    const void *x;                  // [n, H * dim | G * dim | G * vdim], row stride in elements (without cache: H * dim)
    int64_t stride;
    const void *bias;               // as many, or null
    const void *q_norm, *k_norm;    // per head [dim]; whole [H * dim], [G * dim]; null: no norm, or one without a weight
    const float *rope;              // [max_position, 2 * half]: cos | sin
    void *q_out;                    // [n, H * dim]
    void *k_cache, *v_cache;        // flat [num_slots, G * dim], [num_slots, G * vdim]; null: queries only
    const int32_t *slot_mapping;    // [n]
    const int32_t *cu;              // portions: [n_seqs + 1] row bounds
    const int32_t *klen;            // tokens of every sequence once its rows are in (decode: 0 = padded row)
    const int32_t *token_seq;       // portions: sequence of every row
    int64_t num_slots;
    int32_t n, n_seqs, heads, kv_heads, dim, vdim, half, max_position;
    int32_t whole;                  // norms over whole projections
    int32_t unit, unit_values;      // norms without weights: of queries and keys, of every head's values
    float eps;
};

__device__ __forceinline__ int row_position(const QkvArgs &a, int t) {
    if (a.cu == nullptr) return a.klen[t] - 1;
    const int seq = min(max(a.token_seq[t], 0), a.n_seqs - 1);
    return a.klen[seq] - (a.cu[seq + 1] - t);
}

// A workgroup per row, 8 elements per lane; a head takes `lanes` lanes (a power of two, dim / 8 of them at work), a thread
// NP heads' pieces, all kept in registers until the norms are known.
template <typename T, int NP>
__global__ __launch_bounds__(256) void qkv_prepare_kernel(QkvArgs a, int32_t log_lanes, int32_t log_vlanes) {
    __shared__ float sh[2][4];
    const int t = blockIdx.x, tid = threadIdx.x;
    const int pos = row_position(a, t);
    const bool cached = a.k_cache != nullptr;
    const int qk_heads = a.heads + (cached ? a.kv_heads : 0);
    T *q_out = static_cast<T *>(a.q_out) + static_cast<int64_t>(t) * a.heads * a.dim;
    if (pos < 0) {                                           // padded row
        for (int i = tid; i < a.heads * a.dim; i += 256) q_out[i] = Elem<T>::from_f32(0.f);
        return;
    }
    const T *x = static_cast<const T *>(a.x) + t * a.stride;
    const T *bias = static_cast<const T *>(a.bias);
    const int64_t slot = cached ? a.slot_mapping[t] : -1;
    const bool store = slot >= 0 && slot < a.num_slots;
    const int lanes = 1 << log_lanes, at = (tid & (lanes - 1)) * 8, head0 = tid >> log_lanes, step = 256 >> log_lanes;
    float v[NP][8];
    float sq_q = 0.f, sq_k = 0.f;
#pragma unroll
    for (int p = 0; p < NP; ++p) {
        const int h = head0 + p * step;
#pragma unroll
        for (int i = 0; i < 8; ++i) v[p][i] = 0.f;
        if (h < qk_heads && at < a.dim) {
            load_f32<T, 8>(x + h * a.dim + at, v[p]);
            if (bias != nullptr) {
                float b[8];
                load_f32<T, 8>(bias + h * a.dim + at, b);
#pragma unroll
                for (int i = 0; i < 8; ++i) v[p][i] += b[i];
            }
        }
    }
    if (store && a.unit_values) {                            // values, head by head
        const int first = (a.heads + a.kv_heads) * a.dim, vlanes = 1 << log_vlanes, e = (tid & (vlanes - 1)) * 8;
        for (int h = tid >> log_vlanes; h < a.kv_heads; h += 256 >> log_vlanes) {
            float y[8], s = 0.f;
#pragma unroll
            for (int i = 0; i < 8; ++i) y[i] = 0.f;
            if (e < a.vdim) {
                load_f32<T, 8>(x + first + h * a.vdim + e, y);
                if (bias != nullptr) {
                    float b[8];
                    load_f32<T, 8>(bias + first + h * a.vdim + e, b);
#pragma unroll
                    for (int i = 0; i < 8; ++i) y[i] += b[i];
                }
            }
#pragma unroll
            for (int i = 0; i < 8; ++i) s = fmaf(y[i], y[i], s);
            for (int d = 1; d < vlanes; d <<= 1) s += __shfl_xor(s, d, 64);      // (a head's lanes are here together)
            const float rstd = rsqrtf(s / static_cast<float>(a.vdim) + a.eps);
#pragma unroll
            for (int i = 0; i < 8; ++i) y[i] *= rstd;
            if (e < a.vdim) store_f32<T, 8>(static_cast<T *>(a.v_cache) + (slot * a.kv_heads + h) * a.vdim + e, y);
        }
    } else if (store) {                                      // values: a plain copy
        const int first = (a.heads + a.kv_heads) * a.dim, count = a.kv_heads * a.vdim;
        for (int e = tid * 8; e < count; e += 2048) {
            float y[8];
            load_f32<T, 8>(x + first + e, y);
            if (bias != nullptr) {
                float b[8];
                load_f32<T, 8>(bias + first + e, b);
#pragma unroll
                for (int i = 0; i < 8; ++i) y[i] += b[i];
            }
            store_f32<T, 8>(static_cast<T *>(a.v_cache) + slot * count + e, y);
        }
    }
    float rstd_q = 1.f, rstd_k = 1.f;
    if (a.whole) {
#pragma unroll
        for (int p = 0; p < NP; ++p) {
            float s = 0.f;
#pragma unroll
            for (int i = 0; i < 8; ++i) s = fmaf(v[p][i], v[p][i], s);
            if (head0 + p * step < a.heads) sq_q += s;
            else sq_k += s;
        }
        sq_q = wave_sum(sq_q);
        sq_k = wave_sum(sq_k);
        if ((tid & 63) == 0) { sh[0][tid >> 6] = sq_q; sh[1][tid >> 6] = sq_k; }
        __syncthreads();
        rstd_q = rsqrtf(((sh[0][0] + sh[0][1]) + (sh[0][2] + sh[0][3])) / static_cast<float>(a.heads * a.dim) + a.eps);
        rstd_k = rsqrtf(((sh[1][0] + sh[1][1]) + (sh[1][2] + sh[1][3])) / static_cast<float>(a.kv_heads * a.dim) + a.eps);
    }
    const int piece = tid & (lanes - 1), hp = a.half >> 3;
    const bool first_half = piece < hp, turns = piece < 2 * hp;
    float c[8], sn[8];
    if (a.half > 0 && turns) {
        const float *angle = a.rope + static_cast<int64_t>(min(pos, a.max_position - 1)) * (2 * a.half) + (first_half ? piece : piece - hp) * 8;
        load_f32<float, 8>(angle, c);
        load_f32<float, 8>(angle + a.half, sn);
    }
#pragma unroll
    for (int p = 0; p < NP; ++p) {
        const int h = head0 + p * step;
        const bool is_q = h < a.heads, mine = h < qk_heads && at < a.dim;
        const T *w = static_cast<const T *>(is_q ? a.q_norm : a.k_norm);
        if (w != nullptr || a.unit) {
            float rstd = is_q ? rstd_q : rstd_k;
            if (!a.whole) {
                float s = 0.f;
#pragma unroll
                for (int i = 0; i < 8; ++i) s = fmaf(v[p][i], v[p][i], s);
                for (int d = 1; d < lanes; d <<= 1) s += __shfl_xor(s, d, 64);
                rstd = rsqrtf(s / static_cast<float>(a.dim) + a.eps);
            }
            if (w == nullptr) {
#pragma unroll
                for (int i = 0; i < 8; ++i) v[p][i] *= rstd;
            } else if (mine) {
                float g[8];
                load_f32<T, 8>(w + (a.whole ? (is_q ? h : h - a.heads) * a.dim : 0) + at, g);
#pragma unroll
                for (int i = 0; i < 8; ++i) v[p][i] *= rstd * g[i];
            }
        }
        if (hp > 0) {
            const int lane = tid & 63, other = turns ? (first_half ? lane + hp : lane - hp) : lane;
#pragma unroll
            for (int i = 0; i < 8; ++i) {
                const float o = __shfl(v[p][i], other, 64);
                if (turns) v[p][i] = first_half ? v[p][i] * c[i] - o * sn[i] : v[p][i] * c[i] + o * sn[i];
            }
        }
        if (!mine) continue;
        if (is_q) store_f32<T, 8>(q_out + h * a.dim + at, v[p]);
        else if (store) store_f32<T, 8>(static_cast<T *>(a.k_cache) + (slot * a.kv_heads + h - a.heads) * a.dim + at, v[p]);
    }
}

// Any sizes: a workgroup per row, queries and keys in LDS.
template <typename T>
__global__ __launch_bounds__(256) void qkv_prepare_any_kernel(QkvArgs a) {
    extern __shared__ float qkv_smem[];
    __shared__ float sh[2][4];
    const int t = blockIdx.x, tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
    const int pos = row_position(a, t);
    const bool cached = a.k_cache != nullptr;
    const int qk_heads = a.heads + (cached ? a.kv_heads : 0), total = qk_heads * a.dim, queries = a.heads * a.dim;
    float *rstd_of = qkv_smem + total;                       // [qk_heads]
    T *q_out = static_cast<T *>(a.q_out) + static_cast<int64_t>(t) * queries;
    if (pos < 0) {
        for (int i = tid; i < queries; i += 256) q_out[i] = Elem<T>::from_f32(0.f);
        return;
    }
    const T *x = static_cast<const T *>(a.x) + t * a.stride;
    const T *bias = static_cast<const T *>(a.bias);
    const int64_t slot = cached ? a.slot_mapping[t] : -1;
    const bool store = slot >= 0 && slot < a.num_slots;
    auto value = [&](int e) -> float { return Elem<T>::to_f32(x[e]) + (bias != nullptr ? Elem<T>::to_f32(bias[e]) : 0.f); };
    float sq_q = 0.f, sq_k = 0.f;
    for (int e = tid; e < total; e += 256) {
        const float v = value(e);
        qkv_smem[e] = v;
        if (e < queries) sq_q = fmaf(v, v, sq_q);
        else sq_k = fmaf(v, v, sq_k);
    }
    if (store && a.unit_values)
        for (int h = wave; h < a.kv_heads; h += 4) {
            float s = 0.f;
            for (int e = lane; e < a.vdim; e += 64) s = fmaf(value(total + h * a.vdim + e), value(total + h * a.vdim + e), s);
            const float rstd = rsqrtf(wave_sum(s) / static_cast<float>(a.vdim) + a.eps);
            for (int e = lane; e < a.vdim; e += 64)
                static_cast<T *>(a.v_cache)[(slot * a.kv_heads + h) * a.vdim + e] = Elem<T>::from_f32(value(total + h * a.vdim + e) * rstd);
        }
    else if (store)
        for (int e = tid; e < a.kv_heads * a.vdim; e += 256)
            static_cast<T *>(a.v_cache)[slot * a.kv_heads * a.vdim + e] = Elem<T>::from_f32(value(total + e));
    sq_q = wave_sum(sq_q);
    sq_k = wave_sum(sq_k);
    if (lane == 0) { sh[0][wave] = sq_q; sh[1][wave] = sq_k; }
    __syncthreads();
    for (int h = wave; h < qk_heads; h += 4) {
        const int which = h < a.heads ? 0 : 1;
        float s = 0.f;
        int count = a.dim;
        if (a.whole) {
            s = (sh[which][0] + sh[which][1]) + (sh[which][2] + sh[which][3]);
            count = (which == 0 ? a.heads : a.kv_heads) * a.dim;
        } else {
            for (int e = lane; e < a.dim; e += 64) s = fmaf(qkv_smem[h * a.dim + e], qkv_smem[h * a.dim + e], s);
            s = wave_sum(s);
        }
        if (lane == 0) rstd_of[h] = rsqrtf(s / static_cast<float>(count) + a.eps);
    }
    __syncthreads();
    auto normed = [&](int h, int e) -> float {
        const bool is_q = h < a.heads;
        const T *w = static_cast<const T *>(is_q ? a.q_norm : a.k_norm);
        const float v = qkv_smem[h * a.dim + e];
        if (w == nullptr) return a.unit ? v * rstd_of[h] : v;
        return v * (rstd_of[h] * Elem<T>::to_f32(w[(a.whole ? (is_q ? h : h - a.heads) * a.dim : 0) + e]));
    };
    const float *angle = a.half > 0 ? a.rope + static_cast<int64_t>(min(pos, a.max_position - 1)) * (2 * a.half) : nullptr;
    for (int i = tid; i < total; i += 256) {
        const int h = i / a.dim, e = i % a.dim;
        float y = normed(h, e);
        if (e < 2 * a.half) {
            const int k = e < a.half ? e : e - a.half;
            const float o = normed(h, e < a.half ? e + a.half : e - a.half), c = angle[k], s = angle[a.half + k];
            y = e < a.half ? y * c - o * s : y * c + o * s;
        }
        if (h < a.heads) q_out[i] = Elem<T>::from_f32(y);
        else if (store) static_cast<T *>(a.k_cache)[slot * a.kv_heads * a.dim + i - queries] = Elem<T>::from_f32(y);
    }
}

constexpr int kMaxPieces = 8;
constexpr size_t kMaxLds = 150 * 1024;

template <typename T>
static int launch_qkv_prepare(const QkvArgs &a, hipStream_t s) {
    const int qk_heads = a.heads + (a.k_cache ? a.kv_heads : 0);
    int log_lanes = 0, log_vlanes = 0;
    while ((8 << log_lanes) < a.dim) ++log_lanes;
    while ((8 << log_vlanes) < a.vdim) ++log_vlanes;
    const int pieces = log_lanes <= 6 ? ((qk_heads << log_lanes) + 255) / 256 : kMaxPieces + 1;
    const bool vector = a.dim % 8 == 0 && a.vdim % 8 == 0 && a.half % 8 == 0 && a.stride % 8 == 0 && pieces <= kMaxPieces &&
                        (!a.unit_values || log_vlanes <= 6) && aligned16(a.x) &&
                        aligned16(a.bias) && aligned16(a.q_norm) && aligned16(a.k_norm) && aligned16(a.rope) && aligned16(a.q_out) &&
                        aligned16(a.k_cache) && aligned16(a.v_cache);
    const dim3 grid(a.n), block(256);
    if (vector) {
        if (pieces <= 1) hipLaunchKernelGGL((qkv_prepare_kernel<T, 1>), grid, block, 0, s, a, log_lanes, log_vlanes);
        else if (pieces <= 2) hipLaunchKernelGGL((qkv_prepare_kernel<T, 2>), grid, block, 0, s, a, log_lanes, log_vlanes);
        else if (pieces <= 4) hipLaunchKernelGGL((qkv_prepare_kernel<T, 4>), grid, block, 0, s, a, log_lanes, log_vlanes);
        else hipLaunchKernelGGL((qkv_prepare_kernel<T, kMaxPieces>), grid, block, 0, s, a, log_lanes, log_vlanes);
        return launch_status();
    }
    const size_t lds = (static_cast<size_t>(qk_heads) * a.dim + qk_heads) * sizeof(float);
    if (lds > kMaxLds) return NVA_ERR_UNSUPPORTED_GEOMETRY;
    if (lds > 60 * 1024 && hipFuncSetAttribute(reinterpret_cast<const void *>(&qkv_prepare_any_kernel<T>), hipFuncAttributeMaxDynamicSharedMemorySize,
                                               static_cast<int>(lds)) != hipSuccess)
        return NVA_ERR_LAUNCH_FAILED;
    hipLaunchKernelGGL((qkv_prepare_any_kernel<T>), grid, block, lds, s, a);
    return launch_status();
}

}  // namespace nva

extern "C" int nva_qkv_prepare(const void *x, int64_t x_row_stride, const void *bias, const void *q_norm_weight, const void *k_norm_weight,
                               int32_t norms, const float *rope_cache, void *q_out, void *k_cache, void *v_cache,
                               const int32_t *slot_mapping, int64_t num_slots, const int32_t *cu_seqlens_q, const int32_t *seq_lens,
                               const int32_t *token_seq, int32_t n_tokens, int32_t n_seqs, int32_t num_heads, int32_t num_kv_heads,
                               int32_t qk_dim, int32_t v_dim, int32_t rot_dims, int32_t max_position, float eps, int32_t dtype, void *stream) {
    using namespace nva;
    if (n_tokens < 0 || n_seqs < 0 || num_heads <= 0 || num_kv_heads <= 0 || qk_dim <= 0 || v_dim <= 0 || num_slots < 0 || rot_dims < 0 ||
        rot_dims % 2 != 0 || rot_dims > qk_dim || (rot_dims > 0 && max_position <= 0))
        return NVA_ERR_BAD_SHAPE;
    if (!known_dtype(dtype) || (norms & ~(NVA_QKV_NORM_WHOLE | NVA_QKV_NORM_UNIT | NVA_QKV_NORM_VALUES)) != 0) return NVA_ERR_UNSUPPORTED_GEOMETRY;
    if (n_tokens == 0) return NVA_OK;
    if (!x || !q_out || !seq_lens || (rot_dims > 0 && !rope_cache) || (k_cache == nullptr) != (v_cache == nullptr) || (k_cache && !slot_mapping))
        return NVA_ERR_NULL_POINTER;
    if (cu_seqlens_q && (!token_seq || n_seqs == 0)) return NVA_ERR_NULL_POINTER;
    if (!cu_seqlens_q && n_seqs != n_tokens) return NVA_ERR_BAD_SHAPE;
    const int64_t columns = static_cast<int64_t>(num_heads) * qk_dim + (k_cache ? static_cast<int64_t>(num_kv_heads) * (qk_dim + v_dim) : 0);
    if (x_row_stride < columns) return NVA_ERR_BAD_STRIDE;
    if (columns > (1 << 24)) return NVA_ERR_UNSUPPORTED_GEOMETRY;
    QkvArgs a{};
    a.x = x; a.stride = x_row_stride; a.bias = bias; a.q_norm = q_norm_weight; a.k_norm = k_norm_weight; a.rope = rope_cache; a.q_out = q_out;
    a.k_cache = k_cache; a.v_cache = v_cache; a.slot_mapping = slot_mapping; a.cu = cu_seqlens_q; a.klen = seq_lens; a.token_seq = token_seq;
    a.num_slots = num_slots; a.n = n_tokens; a.n_seqs = n_seqs; a.heads = num_heads; a.kv_heads = num_kv_heads; a.dim = qk_dim; a.vdim = v_dim;
    a.half = rot_dims / 2; a.max_position = max_position; a.whole = (norms & NVA_QKV_NORM_WHOLE) != 0; a.unit = (norms & NVA_QKV_NORM_UNIT) != 0;
    a.unit_values = (norms & NVA_QKV_NORM_VALUES) != 0; a.eps = eps;
    hipStream_t s = static_cast<hipStream_t>(stream);
    return dtype == NVA_DTYPE_BF16 ? launch_qkv_prepare<bf16_t>(a, s) : launch_qkv_prepare<float>(a, s);
}
