// Retention: linear attention with one fixed decay per head.
//   S_t = decay S_{t-1} + k_t v_t^T      o_t = S_t^T q_t
// q and k carry rotary positions, k is scaled by dim^-1/2; every head's o is divided by its root mean
// square and multiplied by silu of the gate projection.  The kernels take the projections as they
// come out of the matrix product (rows of q | k | v | gate) and do everything else.  State, rotated q
// and k, decays and norms are fp32; the state lives in slots [slot, head, dim, vdim].
#include "nva_elem.h"

#include <math.h>

namespace nva {

struct RetentionArgs {
    const void *x;                   // [n, 2 H dim + 2 H vdim]: q, k, v, gate
    int64_t stride;                  // elements
    float *state;                    // [num_slots, H, dim, vdim]
    const int32_t *slots;            // [n_seqs]
    const int32_t *cu;               // portions: [n_seqs + 1]; decode: null, row i is sequence i
    const int32_t *klen;             // tokens of every sequence, this step's included (decode: 0 = padded row)
    const int64_t *positions;        // [n]
    const float *rope;               // [max_position, 2 half]: cos | sin
    const float *log2_decay;         // [H]
    void *out;                       // [n, H vdim] dense
    int32_t n, n_seqs, heads, dim, vdim, half, num_slots, max_position;
    float k_scale, eps;
};

// Any sizes, bf16 or fp32, portions and single tokens: one workgroup per (sequence, head) walks the
// tokens; the state stays in its slot (the L2 holds it) and is updated in place.
constexpr int kScanMaxDim = 512;

template <typename T>
__global__ __launch_bounds__(256) void retention_scan_any_kernel(RetentionArgs a) {
    __shared__ float sh_q[kScanMaxDim], sh_k[kScanMaxDim], sh_v[kScanMaxDim], sh_red[kScanMaxDim > 256 ? kScanMaxDim : 256], sh_w[4];
    const int seq = blockIdx.x / a.heads, head = blockIdx.x % a.heads;
    const int tid = threadIdx.x;
    int first = seq, count = 1, start = a.klen[seq] - 1;
    if (a.cu != nullptr) {
        first = a.cu[seq];
        count = a.cu[seq + 1] - first;
        start = a.klen[seq] - count;
    }
    const int slot = a.slots[seq];
    const bool live = start >= 0 && count > 0 && static_cast<uint32_t>(slot) < static_cast<uint32_t>(a.num_slots);
    T *out = static_cast<T *>(a.out);
    if (!live) {                                           // padded row: a defined result, nothing stored
        for (int t = 0; t < count; ++t)
            for (int c = tid; c < a.vdim; c += 256)
                out[(static_cast<int64_t>(first + t) * a.heads + head) * a.vdim + c] = Elem<T>::from_f32(0.f);
        return;
    }
    float *S = a.state + (static_cast<int64_t>(slot) * a.heads + head) * a.dim * a.vdim;
    const float decay = exp2f(a.log2_decay[head]);
    int cols = 1;                                          // threads side by side over the value columns
    while (cols < a.vdim && cols < 256) cols <<= 1;
    const int groups = 256 / cols, c_lane = tid % cols, group = tid / cols;
    const int64_t qk = static_cast<int64_t>(a.heads) * a.dim;
    for (int t = 0; t < count; ++t) {
        const T *row = static_cast<const T *>(a.x) + static_cast<int64_t>(first + t) * a.stride;
        const T *q = row + static_cast<int64_t>(head) * a.dim, *k = q + qk;
        const T *v = row + 2 * qk + static_cast<int64_t>(head) * a.vdim, *gate = v + static_cast<int64_t>(a.heads) * a.vdim;
        const int64_t pos = min(max(a.positions[first + t], static_cast<int64_t>(0)), static_cast<int64_t>(a.max_position) - 1);
        for (int i = tid; i < a.dim; i += 256) {
            float qv = Elem<T>::to_f32(q[i]), kv = Elem<T>::to_f32(k[i]);
            if (i < 2 * a.half) {
                const bool lower = i < a.half;
                const int f = lower ? i : i - a.half, other = lower ? i + a.half : i - a.half;
                const float c = a.rope[pos * (2 * a.half) + f], s = a.rope[pos * (2 * a.half) + a.half + f];
                const float sg = lower ? -s : s;
                qv = qv * c + Elem<T>::to_f32(q[other]) * sg;
                kv = kv * c + Elem<T>::to_f32(k[other]) * sg;
            }
            sh_q[i] = qv;
            sh_k[i] = kv * a.k_scale;
        }
        for (int c = tid; c < a.vdim; c += 256) sh_v[c] = Elem<T>::to_f32(v[c]);
        __syncthreads();
        const bool fresh = start == 0 && t == 0;
        float ss = 0.f;
        for (int c0 = 0; c0 < a.vdim; c0 += cols) {
            const int c = c0 + c_lane;
            float acc = 0.f;
            if (c < a.vdim) {
                const float vc = sh_v[c];
                for (int r = group; r < a.dim; r += groups) {
                    float *p = S + static_cast<int64_t>(r) * a.vdim + c;
                    const float s = fmaf(decay, fresh ? 0.f : *p, sh_k[r] * vc);
                    *p = s;
                    acc = fmaf(s, sh_q[r], acc);
                }
            }
            if (groups == 1) {
                if (c < a.vdim) sh_red[c] = acc;           // (kScanMaxDim columns)
            } else {
                sh_red[tid] = acc;
                __syncthreads();
                if (tid < cols) {
                    for (int g = 1; g < groups; ++g) acc += sh_red[g * cols + tid];
                    sh_red[tid] = acc;
                }
            }
        }
        __syncthreads();
        for (int c = tid; c < a.vdim; c += 256) ss = fmaf(sh_red[c], sh_red[c], ss);
        ss = wave_sum(ss);
        if ((tid & 63) == 0) sh_w[tid >> 6] = ss;
        __syncthreads();
        const float inv = rsqrtf(((sh_w[0] + sh_w[1]) + (sh_w[2] + sh_w[3])) / static_cast<float>(a.vdim) + a.eps);
        for (int c = tid; c < a.vdim; c += 256) {
            const float z = Elem<T>::to_f32(gate[c]);
            out[(static_cast<int64_t>(first + t) * a.heads + head) * a.vdim + c] =
                Elem<T>::from_f32(sh_red[c] * inv * (z * sigmoid_of<T>(z)));
        }
        __syncthreads();
    }
}

template <typename T>
static int launch_scan_any(const RetentionArgs &a, hipStream_t s) {
    hipLaunchKernelGGL((retention_scan_any_kernel<T>), dim3(a.n_seqs * a.heads), dim3(256), 0, s, a);
    return launch_status();
}

}  // namespace nva

extern "C" int nva_retention(const void *qkvg, int64_t row_stride, float *state, const int32_t *state_slots_of_seq,
                             const int32_t *cu_seqlens_q, const int32_t *seq_lens, const int64_t *positions,
                             const float *rope_cache, const float *log2_decay, void *out, int32_t n_tokens, int32_t n_seqs,
                             int32_t max_seqlen_q, int32_t num_heads, int32_t qk_dim, int32_t v_dim, int32_t rot_dims,
                             int32_t max_position, int32_t num_state_slots, float k_scale, float eps, int32_t dtype,
                             void *stream) {
    using namespace nva;
    if (n_tokens < 0 || n_seqs < 0 || max_seqlen_q < 0 || num_heads <= 0 || qk_dim <= 0 || v_dim <= 0 || rot_dims < 0 ||
        rot_dims > qk_dim || max_position <= 0 || num_state_slots < 0)
        return NVA_ERR_BAD_SHAPE;
    if (rot_dims % 2 != 0 || qk_dim > kScanMaxDim || v_dim > kScanMaxDim || !known_dtype(dtype)) return NVA_ERR_UNSUPPORTED_GEOMETRY;
    if (n_tokens == 0 || n_seqs == 0) return NVA_OK;
    if (!qkvg || !state || !state_slots_of_seq || !seq_lens || !positions || !log2_decay || !out) return NVA_ERR_NULL_POINTER;
    if (rot_dims > 0 && !rope_cache) return NVA_ERR_NULL_POINTER;
    if (cu_seqlens_q == nullptr && n_seqs != n_tokens) return NVA_ERR_BAD_SHAPE;
    if (row_stride < 2 * static_cast<int64_t>(num_heads) * (qk_dim + v_dim)) return NVA_ERR_BAD_STRIDE;
    if (static_cast<int64_t>(n_seqs) * num_heads > 0x7fffffffLL) return NVA_ERR_BAD_SHAPE;
    RetentionArgs a{};
    a.x = qkvg; a.stride = row_stride; a.state = state; a.slots = state_slots_of_seq; a.cu = cu_seqlens_q; a.klen = seq_lens;
    a.positions = positions; a.rope = rope_cache; a.log2_decay = log2_decay; a.out = out; a.n = n_tokens; a.n_seqs = n_seqs;
    a.heads = num_heads; a.dim = qk_dim; a.vdim = v_dim; a.half = rot_dims / 2; a.num_slots = num_state_slots;
    a.max_position = max_position; a.k_scale = k_scale; a.eps = eps;
    hipStream_t s = static_cast<hipStream_t>(stream);
    return dtype == NVA_DTYPE_BF16 ? launch_scan_any<bf16_t>(a, s) : launch_scan_any<float>(a, s);
}
