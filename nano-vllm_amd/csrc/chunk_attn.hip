// Softmax attention over position chunks, keys and values in the paged cache: the query at position p
// sees the keys [floor(p / chunk) * chunk, p] of its own sequence.  Scores may be capped
// (cap * tanh(s / cap)); query/key and value sizes may differ; scores, weights and sums are fp32.
#include "nva_elem.h"

#include <math.h>

namespace nva {

struct ChunkAttnArgs {
    const void *q;                   // [n, H, dim]
    int64_t q_stride;                // elements
    const void *k_cache, *v_cache;   // [num_blocks, block, G, dim], [num_blocks, block, G, vdim]
    const int32_t *block_tables;     // [n_seqs, >= max_blocks]
    int64_t bt_stride;
    const int32_t *cu;               // portions: [n_seqs + 1] row bounds; decode: null, row i is sequence i
    const int32_t *klen;             // tokens of every sequence, this step's included (decode: 0 = padded row)
    const int32_t *token_seq;        // portions: sequence of every row
    void *out;                       // [n, H, vdim] dense
    int32_t n, n_seqs, heads, kv_heads, dim, vdim, block_shift, num_blocks, max_blocks, chunk;
    float scale, cap;                // cap <= 0: none
};

// One wavefront per (row, head), any sizes, bf16 or fp32: lanes are keys for the scores and value
// columns for the weighted sum; running maximum and sum per block of 64 keys.
constexpr int kAnyMaxDim = 512;

template <typename T>
__global__ __launch_bounds__(256) void chunk_attn_any_kernel(ChunkAttnArgs a) {
    __shared__ float sh_q[4][kAnyMaxDim];
    const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
    const int64_t item = static_cast<int64_t>(blockIdx.x) * 4 + wave;
    const bool live = item < static_cast<int64_t>(a.n) * a.heads;
    const int64_t t = live ? item / a.heads : 0;
    const int head = live ? static_cast<int>(item % a.heads) : 0;
    int seq, pos;
    if (a.cu == nullptr) {
        seq = static_cast<int>(t);
        pos = a.klen[seq] - 1;
    } else {
        seq = min(max(a.token_seq[t], 0), a.n_seqs - 1);
        pos = a.klen[seq] - (a.cu[seq + 1] - static_cast<int>(t));
    }
    if (live) {
        const T *q = static_cast<const T *>(a.q) + t * a.q_stride + static_cast<int64_t>(head) * a.dim;
        for (int i = lane; i < a.dim; i += 64) sh_q[wave][i] = Elem<T>::to_f32(q[i]);
    }
    __syncthreads();
    if (!live) return;
    const int g = head / (a.heads / a.kv_heads);
    const int lo = pos < 0 ? 0 : pos / a.chunk * a.chunk;
    float m = -INFINITY, sum = 0.f;
    float acc[kAnyMaxDim / 64];
#pragma unroll
    for (int i = 0; i < kAnyMaxDim / 64; ++i) acc[i] = 0.f;
    const int bmask = (1 << a.block_shift) - 1;
    for (int j0 = lo; j0 <= pos; j0 += 64) {
        const int j = j0 + lane;
        int64_t row = -1;                                  // cache row of this lane's key
        if (j <= pos && (j >> a.block_shift) < a.max_blocks) {
            const int blk = a.block_tables[seq * a.bt_stride + (j >> a.block_shift)];
            if (static_cast<uint32_t>(blk) < static_cast<uint32_t>(a.num_blocks))
                row = (static_cast<int64_t>(blk) << a.block_shift) + (j & bmask);
        }
        float s = -INFINITY;
        if (row >= 0) {
            const T *k = static_cast<const T *>(a.k_cache) + (row * a.kv_heads + g) * a.dim;
            float d = 0.f;
            for (int i = 0; i < a.dim; ++i) d = fmaf(sh_q[wave][i], Elem<T>::to_f32(k[i]), d);
            s = d * a.scale;
            if (a.cap > 0.f) s = a.cap * tanh_of<T>(s / a.cap);
        }
        const float m_new = fmaxf(m, wave_max(s));
        if (m_new == -INFINITY) continue;
        const float p = row >= 0 ? exp_of<T>(s - m_new) : 0.f;
        const float keep = m == -INFINITY ? 0.f : exp_of<T>(m - m_new);
        sum = sum * keep + wave_sum(p);
        m = m_new;
#pragma unroll
        for (int i = 0; i < kAnyMaxDim / 64; ++i) acc[i] *= keep;
        const int count = min(64, pos - j0 + 1);
        for (int jj = 0; jj < count; ++jj) {
            const int64_t vrow = __shfl(row, jj, 64);
            if (vrow < 0) continue;
            const float w = __shfl(p, jj, 64);
            const T *v = static_cast<const T *>(a.v_cache) + (vrow * a.kv_heads + g) * a.vdim;
#pragma unroll
            for (int i = 0; i < kAnyMaxDim / 64; ++i)
                if (i * 64 + lane < a.vdim) acc[i] = fmaf(w, Elem<T>::to_f32(v[i * 64 + lane]), acc[i]);
        }
    }
    T *out = static_cast<T *>(a.out) + (t * a.heads + head) * a.vdim;
    const float inv = sum > 0.f ? 1.0f / sum : 0.f;
#pragma unroll
    for (int i = 0; i < kAnyMaxDim / 64; ++i)
        if (i * 64 + lane < a.vdim) out[i * 64 + lane] = Elem<T>::from_f32(acc[i] * inv);
}

template <typename T>
static int launch_any(const ChunkAttnArgs &a, hipStream_t s) {
    const int64_t items = static_cast<int64_t>(a.n) * a.heads;
    hipLaunchKernelGGL((chunk_attn_any_kernel<T>), dim3(static_cast<uint32_t>((items + 3) / 4)), dim3(256), 0, s, a);
    return launch_status();
}

}  // namespace nva

extern "C" int nva_chunk_attn(const void *q, int64_t q_row_stride, const void *k_cache, const void *v_cache,
                              const int32_t *block_tables, int64_t bt_row_stride, int32_t max_blocks,
                              const int32_t *cu_seqlens_q, const int32_t *seq_lens, const int32_t *token_seq, void *out,
                              int32_t n_tokens, int32_t n_seqs, int32_t max_seqlen_q, int32_t num_heads,
                              int32_t num_kv_heads, int32_t qk_dim, int32_t v_dim, int32_t block_size,
                              int32_t num_blocks, int32_t chunk, float scale, float softcap, int32_t dtype,
                              void *stream) {
    using namespace nva;
    if (n_tokens < 0 || n_seqs < 0 || num_heads <= 0 || num_kv_heads <= 0 || qk_dim <= 0 || v_dim <= 0 || num_blocks < 0 ||
        max_blocks < 0 || chunk <= 0 || max_seqlen_q < 0 || num_heads % num_kv_heads != 0)
        return NVA_ERR_BAD_SHAPE;
    const int shift = block_shift_of(block_size);
    if (shift < 0 || qk_dim > kAnyMaxDim || v_dim > kAnyMaxDim || !known_dtype(dtype)) return NVA_ERR_UNSUPPORTED_GEOMETRY;
    if (n_tokens == 0) return NVA_OK;
    if (!q || !k_cache || !v_cache || !block_tables || !seq_lens || !out) return NVA_ERR_NULL_POINTER;
    const bool decode = cu_seqlens_q == nullptr;
    if (!decode && (!token_seq || n_seqs == 0)) return NVA_ERR_NULL_POINTER;
    if (decode && n_seqs != n_tokens) return NVA_ERR_BAD_SHAPE;
    if (q_row_stride < static_cast<int64_t>(num_heads) * qk_dim || bt_row_stride < max_blocks) return NVA_ERR_BAD_STRIDE;
    if (static_cast<int64_t>(n_tokens) * num_heads / 4 > 0x7ffffff0LL) return NVA_ERR_BAD_SHAPE;
    ChunkAttnArgs a{};
    a.q = q; a.q_stride = q_row_stride; a.k_cache = k_cache; a.v_cache = v_cache; a.block_tables = block_tables;
    a.bt_stride = bt_row_stride; a.cu = cu_seqlens_q; a.klen = seq_lens; a.token_seq = token_seq; a.out = out;
    a.n = n_tokens; a.n_seqs = n_seqs; a.heads = num_heads; a.kv_heads = num_kv_heads; a.dim = qk_dim; a.vdim = v_dim;
    a.block_shift = shift; a.num_blocks = num_blocks; a.max_blocks = max_blocks; a.chunk = chunk; a.scale = scale;
    a.cap = softcap;
    hipStream_t s = static_cast<hipStream_t>(stream);
    return dtype == NVA_DTYPE_BF16 ? launch_any<bf16_t>(a, s) : launch_any<float>(a, s);
}
