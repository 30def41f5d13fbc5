// Softmax attention under a mask of positions, keys and values in the paged cache: the query at position p sees the
// keys [first_key(p), p] of its own sequence, where
//   chunks    first_key(p) = floor(p / span) * span
//   window    first_key(p) = max(0, p - span + 1)     (a span no sequence reaches: all earlier keys)
// Scores may be capped (cap * tanh(s / cap)), or lose a bias that grows with the logarithm of the distance (slope
// ln(1 + rate (p - j)), two numbers per head); a head may have a sink, one more score that belongs to no key and only
// enters the sum of the weights; a head's output may be multiplied by sigmoid(gate).  Query/key and value sizes may
// differ; scores, weights and sums are fp32.
#include "nva_elem.h"
#include "nva_matrix.h"

#include <math.h>

#include <algorithm>
#include <type_traits>

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
    int32_t n, n_seqs, heads, kv_heads, dim, vdim, block_shift, num_blocks, max_blocks, span, window;
    float scale, cap;                // cap <= 0: none
    const float *sinks;              // [H] or null
    const float *slope, *rate;       // [H] each or null: distance bias (excludes a cap)
    const void *gate;                // [n, H] logits or null
    int64_t gate_stride;
};

__device__ __forceinline__ int first_key(const ChunkAttnArgs &a, int pos) {
    return a.window ? max(0, pos - a.span + 1) : pos / a.span * a.span;
}
// what a head's output is multiplied by
template <typename T>
__device__ __forceinline__ float head_gate(const ChunkAttnArgs &a, int64_t row, int head) {
    if (a.gate == nullptr) return 1.0f;
    return sigmoid_of<T>(Elem<T>::to_f32(static_cast<const T *>(a.gate)[row * a.gate_stride + head]));
}
constexpr float kLog2e = 1.4426950408889634f;
// the sink's weight where weights are 2^(exponent - top)
__device__ __forceinline__ float sink_weight(const ChunkAttnArgs &a, int head, float top) {
    return a.sinks == nullptr ? 0.f : __builtin_amdgcn_exp2f(fmaf(a.sinks[head], kLog2e, -top));
}

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
    const int lo = pos < 0 ? 0 : first_key(a, pos);
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
            if (a.slope != nullptr) s -= a.slope[head] * log1p_of<T>(a.rate[head] * static_cast<float>(pos - j));
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
    if (a.sinks != nullptr && sum > 0.f) sum += exp_of<T>(a.sinks[head] - m);
    const float inv = sum > 0.f ? head_gate<T>(a, t, head) / sum : 0.f;
#pragma unroll
    for (int i = 0; i < kAnyMaxDim / 64; ++i)
        if (i * 64 + lane < a.vdim) out[i * 64 + lane] = Elem<T>::from_f32(acc[i] * inv);
}

// ---- bf16 on the matrix cores -------------------------------------------------------------------
// Both kernels below compute transposed with v_mfma_f32_16x16x32_bf16: S^T = K Q^T (A: 16 keys x 32 dims,
// B: Q^T), O^T += V^T P^T (A: 16 value columns x 32 keys through LDS transpose reads, B: P^T).  The S^T
// accumulators of two 16-key blocks (register i of lane l: key 4 (l / 16) + i) are a legal key order for
// the second product, so P stays in registers.  The weights are fp32: P goes into the product as the
// sum of two bf16 numbers (its rounding and what the rounding left), 16 bits of mantissa and more, and
// the row sums are taken over the fp32 values.
// Where a score cap of at most kBoundedCap holds, weights need no running maximum: e^{+-cap} and its sums
// stay inside fp32, so nothing is rescaled and partial results of different keys simply add up.

// Otherwise weights need a reference.  For single tokens it is a running maximum.  For portions it is the maximum of the
// first keys that a query meets, and stays: fp32 holds weights of up to 2^kHeadroom above it, so the accumulators are
// never rescaled.  The maximum over all keys is kept beside it; where that passes the headroom the workgroup walks its
// keys a second time with that maximum for the reference.

constexpr float kBoundedCap = 60.0f;
constexpr float kHeadroom = 64.0f;
enum Cap { kNoCap, kBounded, kCapped, kBiased };

// Raw product -> base-2 exponent of the weight.
struct Weighting {
    float in, out;      // cap: exponent = out - 2 out / (1 + 2^{in s}); none: exponent = in s
    bool capped;
};
static Weighting weighting_of(float scale, float cap) {
    if (cap > 0.f) return Weighting{2.0f * kLog2e * scale / cap, kLog2e * cap, true};
    return Weighting{kLog2e * scale, 0.f, false};
}
__device__ __forceinline__ float exponent_of(const Weighting &w, bool capped, float s) {
    if (capped) return fmaf(-2.0f * w.out, __builtin_amdgcn_rcpf(1.0f + __builtin_amdgcn_exp2f(w.in * s)), w.out);
    return w.in * s;
}
// ... minus a distance bias: ahead = 1 + rate * distance
__device__ __forceinline__ float biased_exponent(float in, float s, float slope, float ahead) {
    return fmaf(-slope, __builtin_amdgcn_logf(ahead), in * s);
}

// Portions: a workgroup of four wavefronts takes 4 * 16 * NQ queries of one head and walks the keys that
// any of them sees in tiles of 64, double-buffered in LDS.  DK, DV: sizes the registers are laid out for.
// kDirect (the model's sizes are exactly these): tiles travel global -> LDS without a register in between,
// the LDS image laid out in 1 KB blocks of 16 keys x 32 dims with the 16-byte pieces permuted so that
// operand reads spread over the banks -- the scheme of the prefill kernel for whole contexts, whose
// description gives the permutations.  Otherwise (smaller sizes, multiples of 8) tiles go through registers
// into padded rows, zero-filled to DK and DV.
template <int DK, int DV, int NQ, Cap kCap, bool kDirect>
__global__ __launch_bounds__(256, DK + DV > 256 ? 1 : 2) void chunk_prefill_kernel(const ChunkAttnArgs a, const Weighting w,
                                                                                  const int32_t q_tiles) {
    constexpr int kBM = 64 * NQ, kBN = 64;
    constexpr int kKPitch = DK * 2 + 16, kVPitch = DV * 2 + 32;      // bytes; chosen so that operand reads spread over the banks
    constexpr int kKPieces = DK / 32, kVPieces = DV / 32;           // 16-byte pieces of a tile per thread
    constexpr int kKTile = kDirect ? kBN * DK * 2 : kBN * kKPitch, kVTile = kDirect ? kBN * DV * 2 : kBN * kVPitch;
    __shared__ __attribute__((aligned(1024))) unsigned char smem[2 * (kKTile + kVTile)];
    const lds_char_ptr lds = (lds_char_ptr)(&smem[0]);
    // kv heads fastest, query tiles last to first: as in the prefill kernel for whole contexts, the
    // workgroups that share keys run close together on one XCD
    const int group = a.heads / a.kv_heads;
    const int g_kv = blockIdx.x % a.kv_heads;
    int rest = blockIdx.x / a.kv_heads;
    const int head = g_kv * group + rest % group;
    rest /= group;
    const int row0 = (q_tiles - 1 - rest % q_tiles) * kBM;
    const int seq = rest / q_tiles;
    const int tid = threadIdx.x, lane = tid & 63;
    const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
    const int r = lane & 15, g = lane >> 4;
    const int t0 = a.cu[seq], lq = a.cu[seq + 1] - t0;
    if (row0 >= lq) return;
    const int start = a.klen[seq] - lq;
    if (start < 0) return;
    const int last_row = min(row0 + kBM, lq) - 1;
    const int key_end = start + last_row;                            // last key any query of the tile sees
    const int key_begin = first_key(a, start + row0) & ~(kBN - 1);
    const int ntiles = (key_end - key_begin) / kBN + 1;
    const bf16_t *kc = static_cast<const bf16_t *>(a.k_cache) + static_cast<int64_t>(g_kv) * a.dim;
    const bf16_t *vc = static_cast<const bf16_t *>(a.v_cache) + static_cast<int64_t>(g_kv) * a.vdim;
    const int64_t kstride = static_cast<int64_t>(a.kv_heads) * a.dim, vstride = static_cast<int64_t>(a.kv_heads) * a.vdim;
    const int bmask = (1 << a.block_shift) - 1;

    // queries of this wavefront
    int pos[NQ], lo[NQ];
    u32x4_t qf[NQ][DK / 32];
#pragma unroll
    for (int qa = 0; qa < NQ; ++qa) {
        const int row = row0 + wave * 16 * NQ + 16 * qa + r;
        pos[qa] = start + row;
        lo[qa] = first_key(a, pos[qa]);
        const bf16_t *q = static_cast<const bf16_t *>(a.q) + static_cast<int64_t>(t0 + min(row, lq - 1)) * a.q_stride +
                          static_cast<int64_t>(head) * a.dim + 8 * g;
#pragma unroll
        for (int ks = 0; ks < DK / 32; ++ks) {
            qf[qa][ks] = u32x4_t{0, 0, 0, 0};
            if (32 * ks + 8 * g < a.dim) qf[qa][ks] = *reinterpret_cast<const u32x4_t *>(q + 32 * ks);
        }
    }
    const int w_first = start + row0 + wave * 16 * NQ;               // the wavefront's queries: first and last position
    const int w_last = min(w_first + 16 * NQ - 1, key_end);
    const bool w_live = row0 + wave * 16 * NQ < lq;
    const int w_lo = first_key(a, w_first);                          // oldest key one of them sees
    const int w_lo_all = first_key(a, w_last);                       // keys from here to w_first are seen by all

    // ---- tiles into LDS.  Direct: a tile's block id is asked for one tile ahead (in a vector register, so
    // that nothing waits for it before it is used), its loads go out while the tile before it is multiplied.
    int lane_zero;
    asm volatile("v_mov_b32 %0, 0" : "=v"(lane_zero));
    auto block_of = [&](int tile) __attribute__((always_inline)) -> int {
        const int col = (key_begin + tile * kBN) >> a.block_shift;
        return a.block_tables[seq * a.bt_stride + min(col, a.max_blocks - 1) + lane_zero];
    };
    u32x4_t kreg[kDirect ? 1 : kKPieces], vreg[kDirect ? 1 : kVPieces];
    const int lk16 = lane >> 2, lj = lane & 3;
    const uint32_t lds_k0 = __builtin_amdgcn_readfirstlane(static_cast<uint32_t>(reinterpret_cast<uintptr_t>(lds)) + wave * (DK / 32) * 1024);
    const uint32_t lds_v0 = __builtin_amdgcn_readfirstlane(static_cast<uint32_t>(reinterpret_cast<uintptr_t>(lds)) + 2 * kKTile + wave * (DV / 32) * 1024);
    uint32_t koff = 0, voff = 0;
    auto fetch = [&](int tile, int blk_v, int buf) __attribute__((always_inline)) -> bool {
        const int key0 = key_begin + tile * kBN;
        const int blk = __builtin_amdgcn_readfirstlane(blk_v);
        const bool ok = static_cast<uint32_t>(blk) < static_cast<uint32_t>(a.num_blocks);
        const int64_t base = (static_cast<int64_t>(ok ? blk : 0) << a.block_shift) + (key0 & bmask);
        if constexpr (kDirect) {
            const int row = min(wave * 16 + lk16, key_end - key0);   // rows past the last key repeat it and are masked
            koff = static_cast<uint32_t>(row * kstride + (lj ^ ((0 - (lk16 >> 2)) & 3)) * 8) * 2;
            voff = static_cast<uint32_t>(row * vstride + (lj ^ (2 * ((lk16 >> 2) & 1))) * 8) * 2;
            const char *kb = reinterpret_cast<const char *>(kc + base * kstride), *vb = reinterpret_cast<const char *>(vc + base * vstride);
#pragma unroll
            for (int x = 0; x < DK / 32; ++x) load_to_lds_16(kb + 64 * x, koff, lds_k0 + buf * kKTile + 1024 * x);
#pragma unroll
            for (int x = 0; x < DV / 32; ++x) load_to_lds_16(vb + 64 * x, voff, lds_v0 + buf * kVTile + 1024 * x);
        } else {
#pragma unroll
            for (int i = 0; i < kKPieces; ++i) {
                const int p = i * 256 + tid, row = p / (DK / 8), e = p % (DK / 8) * 8;
                kreg[i] = u32x4_t{0, 0, 0, 0};
                if (ok && key0 + row <= key_end && e < a.dim) kreg[i] = *reinterpret_cast<const u32x4_t *>(kc + (base + row) * kstride + e);
            }
#pragma unroll
            for (int i = 0; i < kVPieces; ++i) {
                const int p = i * 256 + tid, row = p / (DV / 8), e = p % (DV / 8) * 8;
                vreg[i] = u32x4_t{0, 0, 0, 0};
                if (ok && key0 + row <= key_end && e < a.vdim) vreg[i] = *reinterpret_cast<const u32x4_t *>(vc + (base + row) * vstride + e);
            }
        }
        return ok;
    };
    auto put = [&](int buf) __attribute__((always_inline)) {
        if constexpr (kDirect) {
            loads_issued(koff, voff);
            asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
        } else {
            const lds_char_ptr kl = lds + buf * kKTile, vl = lds + 2 * kKTile + buf * kVTile;
#pragma unroll
            for (int i = 0; i < kKPieces; ++i) {
                const int p = i * 256 + tid;
                *(lds_u32x4_ptr)(kl + p / (DK / 8) * kKPitch + p % (DK / 8) * 16) = kreg[i];
            }
#pragma unroll
            for (int i = 0; i < kVPieces; ++i) {
                const int p = i * 256 + tid;
                *(lds_u32x4_ptr)(vl + p / (DV / 8) * kVPitch + p % (DV / 8) * 16) = vreg[i];
            }
        }
    };

    f32x4_t oacc[DV / 16][NQ];
    float lsum[NQ], m[NQ], top[NQ];
#pragma unroll
    for (int qa = 0; qa < NQ; ++qa) m[qa] = top[qa] = -INFINITY;
    const float to_exp2 = kCap == kCapped || kCap == kBiased ? 1.0f : w.in;      // (not kBounded) of a score, capped or biased already where it is
    const float slope = kCap == kBiased ? a.slope[head] : 0.f, rate = kCap == kBiased ? a.rate[head] : 0.f;

    auto attend = [&](auto masked_c, int key0, int buf) __attribute__((always_inline)) {
        constexpr bool kMasked = decltype(masked_c)::value;
        const lds_char_ptr kl = lds + buf * kKTile + (kDirect ? 16 * (4 * r + (g ^ ((0 - (r >> 2)) & 3))) : r * kKPitch + 16 * g);
        const lds_char_ptr vl = lds + 2 * kKTile + buf * kVTile + (4 * g + (r >> 2)) * (kDirect ? 64 : kVPitch) + 8 * (r & 3);
        auto kpiece = [&](int kb, int ks) __attribute__((always_inline)) -> u32x4_t {
            return *(lds_u32x4_ptr)(kl + (kDirect ? (kb * (DK / 32) + ks) * 1024 : kb * 16 * kKPitch + ks * 64));
        };
        auto vpiece = [&](int kb, int db) __attribute__((always_inline)) -> s16x4_t {
            return __builtin_amdgcn_ds_read_tr16_b64_v4i16((lds_s16x4_ptr)(
                vl + (kDirect ? (kb * (DV / 32) + (db >> 1)) * 1024 + 32 * ((g ^ db) & 1) : kb * 16 * kVPitch + 32 * db)));
        };
        f32x4_t sacc[2][NQ];
        auto scores = [&](int kb) __attribute__((always_inline)) {
#pragma unroll
            for (int qa = 0; qa < NQ; ++qa) sacc[kb & 1][qa] = f32x4_t{0.f, 0.f, 0.f, 0.f};
#pragma unroll
            for (int ks = 0; ks < DK / 32; ++ks) {
                const u32x4_t kf = kpiece(kb, ks);
#pragma unroll
                for (int qa = 0; qa < NQ; ++qa) sacc[kb & 1][qa] = mfma16(kf, qf[qa][ks], sacc[kb & 1][qa]);
            }
        };
        auto seen = [&](int qa, int kb, int i) __attribute__((always_inline)) -> bool {
            const int key = key0 + 16 * kb + 4 * g + i;
            return !kMasked || (key >= lo[qa] && key <= pos[qa]);
        };
#pragma unroll
        for (int half = 0; half < 2; ++half) {           // half a tile at a time, and nothing moved across: fewer registers
            __builtin_amdgcn_sched_barrier(0);
            scores(2 * half);
            scores(2 * half + 1);
            if (kCap != kBounded) {
#pragma unroll
                for (int qa = 0; qa < NQ; ++qa) {
                    float mx = -INFINITY;
                    // 1 + rate * distance of the half tile's first key of this lane; later keys are nearer (unseen ones may
                    // give no number, which nothing reads)
                    const float ahead = fmaf(rate, static_cast<float>(pos[qa] - key0 - 32 * half - 4 * g), 1.0f);
#pragma unroll
                    for (int kb2 = 0; kb2 < 2; ++kb2)
#pragma unroll
                        for (int i = 0; i < 4; ++i) {
                            if (kCap == kBiased) sacc[kb2][qa][i] = biased_exponent(w.in, sacc[kb2][qa][i], slope, fmaf(rate, static_cast<float>(-16 * kb2 - i), ahead));
                            if (kCap == kCapped) sacc[kb2][qa][i] = exponent_of(w, true, sacc[kb2][qa][i]);
                            if (seen(qa, 2 * half + kb2, i)) mx = fmaxf(mx, sacc[kb2][qa][i]);
                        }
                    mx *= to_exp2;
                    top[qa] = fmaxf(top[qa], mx);
                    if (__any(m[qa] == -INFINITY && mx > -INFINITY)) {
                        mx = fmaxf(mx, __shfl_xor(mx, 16, 64));
                        mx = fmaxf(mx, __shfl_xor(mx, 32, 64));
                        if (m[qa] == -INFINITY) m[qa] = mx;
                    }
                }
            }
            u32x4_t ph[NQ], pl[NQ];
#pragma unroll
            for (int qa = 0; qa < NQ; ++qa) {
                const float ref = kCap == kBounded || m[qa] == -INFINITY ? 0.f : m[qa];
#pragma unroll
                for (int kb2 = 0; kb2 < 2; ++kb2) {
                    float p[4];
#pragma unroll
                    for (int i = 0; i < 4; ++i) {
                        const float s = sacc[kb2][qa][i];
                        const bool vis = seen(qa, 2 * half + kb2, i);
                        const float x = kCap == kBounded ? exponent_of(w, true, s) : fmaf(s, to_exp2, -ref);
                        p[i] = vis ? __builtin_amdgcn_exp2f(x) : 0.f;
                        lsum[qa] += p[i];
                    }
                    uint32_t h0, l0, h1, l1;
                    split_pair(p[0], p[1], h0, l0);
                    split_pair(p[2], p[3], h1, l1);
                    ph[qa][2 * kb2] = h0; ph[qa][2 * kb2 + 1] = h1;
                    pl[qa][2 * kb2] = l0; pl[qa][2 * kb2 + 1] = l1;
                }
            }
#pragma unroll
            for (int db = 0; db < DV / 16; ++db) {
                const s16x4_t v0 = vpiece(2 * half, db), v1 = vpiece(2 * half + 1, db);
                const u32x4_t vf = __builtin_bit_cast(u32x4_t, __builtin_shufflevector(v0, v1, 0, 1, 2, 3, 4, 5, 6, 7));
#pragma unroll
                for (int qa = 0; qa < NQ; ++qa) {
                    oacc[db][qa] = mfma16(vf, ph[qa], oacc[db][qa]);
                    oacc[db][qa] = mfma16(vf, pl[qa], oacc[db][qa]);
                }
            }
        }
    };

    for (int pass = 0;; ++pass) {
#pragma unroll
        for (int qa = 0; qa < NQ; ++qa) {
            lsum[qa] = 0.f;
#pragma unroll
            for (int db = 0; db < DV / 16; ++db) oacc[db][qa] = f32x4_t{0.f, 0.f, 0.f, 0.f};
        }
        int blk_next = block_of(1);
        bool ok = fetch(0, block_of(0), 0);
        put(0);
        __syncthreads();
        for (int tile = 0; tile < ntiles; ++tile) {
            const int buf = tile & 1;
            bool ok_next = false;
            if (tile + 1 < ntiles) {
                ok_next = fetch(tile + 1, blk_next, buf ^ 1);        // (that buffer was read one tile ago, a barrier lies between)
                blk_next = block_of(tile + 2);
            }
            const int key0 = key_begin + tile * kBN;
            if (ok && w_live && key0 <= w_last && key0 + kBN > w_lo) {
                if (key0 >= w_lo_all && key0 + kBN - 1 <= w_first) attend(std::false_type{}, key0, buf);
                else attend(std::true_type{}, key0, buf);
            }
            if (tile + 1 < ntiles) put(buf ^ 1);
            ok = ok_next;
            __syncthreads();
        }
        if (kCap == kBounded || pass > 0) break;
        bool again = false;
#pragma unroll
        for (int qa = 0; qa < NQ; ++qa) again |= top[qa] > m[qa] + kHeadroom;
        if (!__syncthreads_or(again)) break;
#pragma unroll
        for (int qa = 0; qa < NQ; ++qa) {
            float mx = fmaxf(top[qa], __shfl_xor(top[qa], 16, 64));
            m[qa] = fmaxf(mx, __shfl_xor(mx, 32, 64));
        }
    }
    if (!w_live) return;
#pragma unroll
    for (int qa = 0; qa < NQ; ++qa) {
        float l = lsum[qa];
        l += __shfl_xor(l, 16, 64);
        l += __shfl_xor(l, 32, 64);
        const int row = row0 + wave * 16 * NQ + 16 * qa + r;
        if (row >= lq) continue;
        l += sink_weight(a, head, kCap == kBounded ? 0.f : m[qa]);
        const float inv = l > 0.f ? head_gate<bf16_t>(a, t0 + row, head) / l : 0.f;
        bf16_t *out = static_cast<bf16_t *>(a.out) + (static_cast<int64_t>(t0 + row) * a.heads + head) * a.vdim + 4 * g;
#pragma unroll
        for (int db = 0; db < DV / 16; ++db)
            if (16 * db + 4 * g < a.vdim) {
                const f32x4_t o = oacc[db][qa];
                *reinterpret_cast<u32x2_t *>(out + 16 * db) = u32x2_t{pack_bf16x2(o[0] * inv, o[1] * inv), pack_bf16x2(o[2] * inv, o[3] * inv)};
            }
    }
}

// Single tokens: a workgroup takes one (sequence, kv head, range of keys), its wavefronts tiles of 32 keys
// in turn; up to 16 query heads of the kv head are the columns of the products.  K goes from memory
// straight into operand registers, V through wavefront-private LDS for the transpose.  The four wavefronts
// meet in LDS; with more than one range per pair the results are partial (fp32 sums with their
// weights' sum and reference) and chunk_merge_kernel adds them up.
struct SplitArgs {
    float *partials;         // [n, splits, heads, vdim + 2]: sums, sum of the weights, reference exponent
    int32_t splits, keys;    // ranges per sequence, keys per range (a multiple of 128)
    int32_t head_groups;     // groups of 16 query heads per kv head
};

template <int DK, int DV, Cap kCap>
__global__ __launch_bounds__(256, DK + DV > 256 ? 1 : 3) void chunk_decode_kernel(const ChunkAttnArgs a, const Weighting w, const SplitArgs sp) {
    constexpr bool kPlain = kCap == kBounded;            // (kCapped: with or without a cap)
    constexpr int kVPitch = DV * 2 + 32;
    constexpr int kWaveBytes = 32 * kVPitch > 16 * DV * 4 ? 32 * kVPitch : 16 * DV * 4;
    constexpr int kVPieces = DV / 16;                    // 16-byte pieces of a 32-key V tile per lane
    __shared__ __attribute__((aligned(16))) unsigned char smem[4 * kWaveBytes];
    __shared__ float sh_l[4][16], sh_m[4][16];
    const int tid = threadIdx.x, lane = tid & 63;
    const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
    const int r = lane & 15, g = lane >> 4;
    // Workgroups are handed out in order, round-robin over XCDs and their CUs: sequences are the fastest index, so
    // that ranges past the end of short sequences do not fall on the same CUs again and again (with the
    // ranges of a sequence next to one another half the machine idled at four ranges)
    const int seq = blockIdx.x % a.n;
    int rest = blockIdx.x / a.n;
    const int split = rest % sp.splits;
    rest /= sp.splits;
    const int g_kv = rest % a.kv_heads, hg = rest / a.kv_heads;
    const int group = a.heads / a.kv_heads;
    const int head0 = g_kv * group + hg * 16, nheads = min(16, group - hg * 16);
    const int pos = a.klen[seq] - 1;
    bf16_t *out = static_cast<bf16_t *>(a.out) + (static_cast<int64_t>(seq) * a.heads + head0) * a.vdim;
    if (pos < 0) {
        if (sp.splits == 1)
            for (int i = tid; i < nheads * a.vdim; i += 256) out[i] = 0;
        return;
    }
    const int lo = first_key(a, pos), first = (lo & ~31) + split * sp.keys;
    const int last = min(pos, first + sp.keys - 1);      // last key of this range
    if (first > last) return;
    const int ntiles = (last - first) / 32 + 1;
    const bf16_t *kc = static_cast<const bf16_t *>(a.k_cache) + static_cast<int64_t>(g_kv) * a.dim;
    const bf16_t *vc = static_cast<const bf16_t *>(a.v_cache) + static_cast<int64_t>(g_kv) * a.vdim;
    const int64_t kstride = static_cast<int64_t>(a.kv_heads) * a.dim, vstride = static_cast<int64_t>(a.kv_heads) * a.vdim;
    const int bmask = (1 << a.block_shift) - 1;
    const lds_char_ptr vlds = (lds_char_ptr)(&smem[0]) + wave * kWaveBytes;

    auto block_of = [&](int tile) __attribute__((always_inline)) -> int {
        const int col = (first + tile * 32) >> a.block_shift;
        return tile < ntiles && col < a.max_blocks ? a.block_tables[seq * a.bt_stride + col] : -1;
    };
    u32x4_t kreg[2][DK / 32], vreg[kVPieces];
    auto fetch = [&](int tile, int blk) __attribute__((always_inline)) {
        const int key0 = first + tile * 32;
        const bool ok = static_cast<uint32_t>(blk) < static_cast<uint32_t>(a.num_blocks);
        const int64_t base = (static_cast<int64_t>(ok ? blk : 0) << a.block_shift) + (key0 & bmask);
#pragma unroll
        for (int kb = 0; kb < 2; ++kb) {
            const int row = 16 * kb + r;
            const bf16_t *k = kc + (base + row) * kstride + 8 * g;
#pragma unroll
            for (int ks = 0; ks < DK / 32; ++ks) {
                kreg[kb][ks] = u32x4_t{0, 0, 0, 0};
                if (ok && key0 + row <= last && 32 * ks + 8 * g < a.dim)
                    kreg[kb][ks] = __builtin_nontemporal_load(reinterpret_cast<const u32x4_t *>(k + 32 * ks));
            }
        }
#pragma unroll
        for (int i = 0; i < kVPieces; ++i) {
            const int p = i * 64 + lane, row = p / (DV / 8), e = p % (DV / 8) * 8;
            vreg[i] = u32x4_t{0, 0, 0, 0};
            if (ok && key0 + row <= last && e < a.vdim)
                vreg[i] = __builtin_nontemporal_load(reinterpret_cast<const u32x4_t *>(vc + (base + row) * vstride + e));
        }
    };
    int tile = wave;
    int blk = block_of(tile), blk_next = block_of(tile + 4);
    if (tile < ntiles) fetch(tile, blk);
    u32x4_t qf[DK / 32];
    {
        const bf16_t *q = static_cast<const bf16_t *>(a.q) + static_cast<int64_t>(seq) * a.q_stride +
                          static_cast<int64_t>(head0 + min(r, nheads - 1)) * a.dim + 8 * g;
#pragma unroll
        for (int ks = 0; ks < DK / 32; ++ks) {
            qf[ks] = u32x4_t{0, 0, 0, 0};
            if (32 * ks + 8 * g < a.dim) qf[ks] = *reinterpret_cast<const u32x4_t *>(q + 32 * ks);
        }
    }
    f32x4_t oacc[DV / 16];
#pragma unroll
    for (int db = 0; db < DV / 16; ++db) oacc[db] = f32x4_t{0.f, 0.f, 0.f, 0.f};
    float lsum = 0.f, m = -INFINITY;
    const float slope = kCap == kBiased ? a.slope[head0 + min(r, nheads - 1)] : 0.f, rate = kCap == kBiased ? a.rate[head0 + min(r, nheads - 1)] : 0.f;
    const lds_char_ptr vl = vlds + (4 * g + (r >> 2)) * kVPitch + 8 * (r & 3);
    for (; tile < ntiles; tile += 4) {
        const int key0 = first + tile * 32;
        const bool ok = static_cast<uint32_t>(blk) < static_cast<uint32_t>(a.num_blocks);
#pragma unroll
        for (int i = 0; i < kVPieces; ++i) {
            const int p = i * 64 + lane;
            *(lds_u32x4_ptr)(vlds + p / (DV / 8) * kVPitch + p % (DV / 8) * 16) = vreg[i];
        }
        f32x4_t s[2];
#pragma unroll
        for (int kb = 0; kb < 2; ++kb) {
            s[kb] = f32x4_t{0.f, 0.f, 0.f, 0.f};
#pragma unroll
            for (int ks = 0; ks < DK / 32; ++ks) s[kb] = mfma16(kreg[kb][ks], qf[ks], s[kb]);
        }
        const int blk_this = blk_next;                   // of tile + 4
        blk_next = block_of(tile + 8);
        if (tile + 4 < ntiles) fetch(tile + 4, blk_this);
        blk = blk_this;
        float x[2][4], mx = -INFINITY;
        bool vis[2][4];
        const float ahead = fmaf(rate, static_cast<float>(pos - key0 - 4 * g), 1.0f);      // of this lane's first key, as in the other kernel
#pragma unroll
        for (int kb = 0; kb < 2; ++kb)
#pragma unroll
            for (int i = 0; i < 4; ++i) {
                const int key = key0 + 16 * kb + 4 * g + i;
                vis[kb][i] = ok && key >= lo && key <= last;
                if (kCap == kBiased) x[kb][i] = biased_exponent(w.in, s[kb][i], slope, fmaf(rate, static_cast<float>(-16 * kb - i), ahead));
                else x[kb][i] = exponent_of(w, kPlain || w.capped, s[kb][i]);
                if (vis[kb][i]) mx = fmaxf(mx, x[kb][i]);
            }
        float ref = 0.f;
        if (!kPlain) {
            mx = fmaxf(mx, __shfl_xor(mx, 16, 64));
            mx = fmaxf(mx, __shfl_xor(mx, 32, 64));
            const float m_new = fmaxf(m, mx);
            const float keep = m == -INFINITY ? 0.f : __builtin_amdgcn_exp2f(m - m_new);
            m = m_new;
            ref = m_new == -INFINITY ? 0.f : m_new;
            lsum *= keep;
#pragma unroll
            for (int db = 0; db < DV / 16; ++db)
#pragma unroll
                for (int i = 0; i < 4; ++i) oacc[db][i] *= keep;
        }
        u32x4_t ph, pl;
#pragma unroll
        for (int kb = 0; kb < 2; ++kb) {
            float p[4];
#pragma unroll
            for (int i = 0; i < 4; ++i) {
                p[i] = vis[kb][i] ? __builtin_amdgcn_exp2f(x[kb][i] - ref) : 0.f;
                lsum += p[i];
            }
            uint32_t h0, l0, h1, l1;
            split_pair(p[0], p[1], h0, l0);
            split_pair(p[2], p[3], h1, l1);
            ph[2 * kb] = h0; ph[2 * kb + 1] = h1;
            pl[2 * kb] = l0; pl[2 * kb + 1] = l1;
        }
        // (wavefront-private LDS: in order within the wavefront, no barrier)
#pragma unroll
        for (int db = 0; db < DV / 16; ++db) {
            const s16x4_t v0 = __builtin_amdgcn_ds_read_tr16_b64_v4i16((lds_s16x4_ptr)(vl + 32 * db));
            const s16x4_t v1 = __builtin_amdgcn_ds_read_tr16_b64_v4i16((lds_s16x4_ptr)(vl + 16 * kVPitch + 32 * db));
            const u32x4_t vf = __builtin_bit_cast(u32x4_t, __builtin_shufflevector(v0, v1, 0, 1, 2, 3, 4, 5, 6, 7));
            oacc[db] = mfma16(vf, ph, oacc[db]);
            oacc[db] = mfma16(vf, pl, oacc[db]);
        }
    }
    lsum += __shfl_xor(lsum, 16, 64);
    lsum += __shfl_xor(lsum, 32, 64);
    if (g == 0) { sh_l[wave][r] = lsum; sh_m[wave][r] = m; }
    // the wavefront's sums over its own V tile (read for the last time above)
    float *osh = reinterpret_cast<float *>(&smem[wave * kWaveBytes]);
#pragma unroll
    for (int db = 0; db < DV / 16; ++db) *reinterpret_cast<f32x4_t *>(osh + r * DV + 16 * db + 4 * g) = oacc[db];
    __syncthreads();
    for (int i = tid; i < nheads * a.vdim; i += 256) {
        const int h = i / a.vdim, c = i % a.vdim;
        float top = 0.f, l = 0.f, o = 0.f;
        if (!kPlain) top = fmaxf(fmaxf(sh_m[0][h], sh_m[1][h]), fmaxf(sh_m[2][h], sh_m[3][h]));
#pragma unroll
        for (int v = 0; v < 4; ++v) {
            const float f = kPlain ? 1.0f : (sh_m[v][h] == -INFINITY ? 0.f : __builtin_amdgcn_exp2f(sh_m[v][h] - top));
            l = fmaf(sh_l[v][h], f, l);
            o = fmaf(reinterpret_cast<const float *>(&smem[v * kWaveBytes])[h * DV + c], f, o);
        }
        if (sp.splits == 1) {
            l += sink_weight(a, head0 + h, top);
            out[i] = f32_to_bf16(l > 0.f ? o * head_gate<bf16_t>(a, seq, head0 + h) / l : 0.f);
        } else {
            float *part = sp.partials + ((static_cast<int64_t>(seq) * sp.splits + split) * a.heads + head0 + h) * (a.vdim + 2);
            part[c] = o;
            if (c == 0) { part[a.vdim] = l; part[a.vdim + 1] = kPlain ? 0.f : top; }
        }
    }
}

// One wavefront per (row, head): adds the partial results of the ranges that hold keys.
__global__ __launch_bounds__(256) void chunk_merge_kernel(const ChunkAttnArgs a, const SplitArgs sp) {
    const int lane = threadIdx.x & 63;
    const int64_t item = static_cast<int64_t>(blockIdx.x) * 4 + (threadIdx.x >> 6);
    if (item >= static_cast<int64_t>(a.n) * a.heads) return;
    const int seq = static_cast<int>(item / a.heads), head = static_cast<int>(item % a.heads);
    const int pos = a.klen[seq] - 1;
    bf16_t *out = static_cast<bf16_t *>(a.out) + item * a.vdim;
    const int lo = pos < 0 ? 0 : first_key(a, pos) & ~31;
    const int count = pos < 0 ? 0 : min(sp.splits, (pos - lo) / sp.keys + 1);
    const int pitch = a.vdim + 2;
    const float *part = sp.partials + (static_cast<int64_t>(seq) * sp.splits * a.heads + head) * pitch;
    const int64_t step = static_cast<int64_t>(a.heads) * pitch;
    // lane j holds sum and reference of range j (up to 64 ranges)
    const float my_l = lane < count ? part[lane * step + a.vdim] : 0.f;
    const float my_m = lane < count ? part[lane * step + a.vdim + 1] : -INFINITY;
    const float top = wave_max(my_m);
    const float f = my_m == -INFINITY ? 0.f : __builtin_amdgcn_exp2f(my_m - top);
    float l = wave_sum(my_l * f);
    if (count > 0) l += sink_weight(a, head, top);
    const float inv = l > 0.f ? head_gate<bf16_t>(a, seq, head) / l : 0.f;
    for (int c = lane; c < a.vdim; c += 64) {
        float o = 0.f;
        for (int j = 0; j < count; ++j) o = fmaf(part[j * step + c], __shfl(f, j, 64), o);
        out[c] = f32_to_bf16(o * inv);
    }
}

// How the keys of a decode step are split: ranges of 512 keys, longer ones where that would be more than 64.
// Depends on shapes only.
static SplitArgs plan_splits(int32_t heads, int32_t kv_heads, int32_t max_blocks, int32_t block_size, int32_t span) {
    SplitArgs sp{};
    sp.head_groups = (heads / kv_heads + 15) / 16;
    const int64_t most = std::min(static_cast<int64_t>(span), static_cast<int64_t>(max_blocks) * block_size) + 31;   // keys one query can see, from a multiple of 32 on
    int64_t keys = std::max(static_cast<int64_t>(512), (most + 63) / 64);
    keys = (keys + 127) / 128 * 128;
    sp.keys = static_cast<int32_t>(keys);
    sp.splits = static_cast<int32_t>(std::max(static_cast<int64_t>(1), (most + keys - 1) / keys));
    return sp;
}

template <int DK, int DV>
static int launch_matrix(const ChunkAttnArgs &a, const SplitArgs &sp, int32_t max_q, hipStream_t s) {
    const bool bounded = a.cap > 0.f && a.cap <= kBoundedCap;
    const Weighting w = weighting_of(a.scale, a.cap);
    if (a.cu == nullptr) {
        const int64_t wgs = static_cast<int64_t>(a.n) * sp.splits * sp.head_groups * a.kv_heads;
        if (wgs > 0x7fffffffLL) return NVA_ERR_BAD_SHAPE;
        const dim3 grid(static_cast<uint32_t>(wgs)), block(256);
        if (a.slope) hipLaunchKernelGGL((chunk_decode_kernel<DK, DV, kBiased>), grid, block, 0, s, a, w, sp);
        else if (bounded) hipLaunchKernelGGL((chunk_decode_kernel<DK, DV, kBounded>), grid, block, 0, s, a, w, sp);
        else hipLaunchKernelGGL((chunk_decode_kernel<DK, DV, kCapped>), grid, block, 0, s, a, w, sp);
        const int rc = launch_status();
        if (rc != NVA_OK || sp.splits == 1) return rc;
        hipLaunchKernelGGL(chunk_merge_kernel, dim3(static_cast<uint32_t>((static_cast<int64_t>(a.n) * a.heads + 3) / 4)), block, 0, s, a, sp);
        return launch_status();
    }
    constexpr int NQ = DK > 128 || DV > 128 ? 1 : 2;
    const int32_t q_tiles = (max_q + 64 * NQ - 1) / (64 * NQ);
    const int64_t wgs = static_cast<int64_t>(a.n_seqs) * q_tiles * a.heads;
    if (wgs > 0x7fffffffLL) return NVA_ERR_BAD_SHAPE;
    if (wgs == 0) return NVA_OK;
    const dim3 grid(static_cast<uint32_t>(wgs)), block(256);
    const bool direct = a.dim == DK && a.vdim == DV;
    if (a.slope && direct) hipLaunchKernelGGL((chunk_prefill_kernel<DK, DV, NQ, kBiased, true>), grid, block, 0, s, a, w, q_tiles);
    else if (a.slope) hipLaunchKernelGGL((chunk_prefill_kernel<DK, DV, NQ, kBiased, false>), grid, block, 0, s, a, w, q_tiles);
    else if (a.cap > 0.f && !bounded) hipLaunchKernelGGL((chunk_prefill_kernel<DK, DV, NQ, kCapped, false>), grid, block, 0, s, a, w, q_tiles);
    else if (bounded && direct) hipLaunchKernelGGL((chunk_prefill_kernel<DK, DV, NQ, kBounded, true>), grid, block, 0, s, a, w, q_tiles);
    else if (bounded) hipLaunchKernelGGL((chunk_prefill_kernel<DK, DV, NQ, kBounded, false>), grid, block, 0, s, a, w, q_tiles);
    else if (direct) hipLaunchKernelGGL((chunk_prefill_kernel<DK, DV, NQ, kNoCap, true>), grid, block, 0, s, a, w, q_tiles);
    else hipLaunchKernelGGL((chunk_prefill_kernel<DK, DV, NQ, kNoCap, false>), grid, block, 0, s, a, w, q_tiles);
    return launch_status();
}

template <int DK>
static int launch_matrix_dk(const ChunkAttnArgs &a, const SplitArgs &sp, int32_t max_q, hipStream_t s) {
    if (a.vdim <= 64) return launch_matrix<DK, 64>(a, sp, max_q, s);
    if (a.vdim <= 128) return launch_matrix<DK, 128>(a, sp, max_q, s);
    return launch_matrix<DK, 256>(a, sp, max_q, s);
}

static bool matrix_ok(const ChunkAttnArgs &a) {
    return a.scale >= 0.f && a.dim % 8 == 0 && a.vdim % 8 == 0 && a.dim <= 256 && a.vdim <= 256 && a.q_stride % 8 == 0 && aligned16(a.q) &&
           aligned16(a.k_cache) && aligned16(a.v_cache) && aligned16(a.out);
}

template <typename T>
static int launch_any(const ChunkAttnArgs &a, hipStream_t s) {
    const int64_t items = static_cast<int64_t>(a.n) * a.heads;
    hipLaunchKernelGGL((chunk_attn_any_kernel<T>), dim3(static_cast<uint32_t>((items + 3) / 4)), dim3(256), 0, s, a);
    return launch_status();
}

}  // namespace nva

extern "C" size_t nva_chunk_attn_workspace_bytes(int32_t n_tokens, int32_t num_heads, int32_t num_kv_heads, int32_t v_dim,
                                                 int32_t max_blocks, int32_t block_size, int32_t chunk) {
    if (n_tokens <= 0 || num_heads <= 0 || num_kv_heads <= 0 || v_dim <= 0 || max_blocks < 0 || block_size <= 0 || chunk <= 0) return 0;
    const nva::SplitArgs sp = nva::plan_splits(num_heads, num_kv_heads, max_blocks, block_size, chunk);
    if (sp.splits == 1) return 0;
    return static_cast<size_t>(n_tokens) * sp.splits * num_heads * (v_dim + 2) * sizeof(float);
}

extern "C" int nva_masked_attn(const void *q, int64_t q_row_stride, const void *k_cache, const void *v_cache,
                              const int32_t *block_tables, int64_t bt_row_stride, int32_t max_blocks,
                              const int32_t *cu_seqlens_q, const int32_t *seq_lens, const int32_t *token_seq, void *out,
                              void *workspace, size_t workspace_bytes, int32_t n_tokens, int32_t n_seqs, int32_t max_seqlen_q, int32_t num_heads,
                              int32_t num_kv_heads, int32_t qk_dim, int32_t v_dim, int32_t block_size,
                              int32_t num_blocks, int32_t mask, int32_t span, float scale, float softcap, const float *sinks,
                              const float *bias_slope, const float *bias_rate, const void *gate, int64_t gate_row_stride, int32_t dtype,
                              void *stream) {
    using namespace nva;
    if (n_tokens < 0 || n_seqs < 0 || num_heads <= 0 || num_kv_heads <= 0 || qk_dim <= 0 || v_dim <= 0 || num_blocks < 0 ||
        max_blocks < 0 || span <= 0 || max_seqlen_q < 0 || num_heads % num_kv_heads != 0)
        return NVA_ERR_BAD_SHAPE;
    const int shift = block_shift_of(block_size);
    if (shift < 0 || (mask != NVA_MASK_CHUNKS && mask != NVA_MASK_WINDOW) || qk_dim > kAnyMaxDim || v_dim > kAnyMaxDim || !known_dtype(dtype)) return NVA_ERR_UNSUPPORTED_GEOMETRY;
    if (bias_slope && softcap > 0.f) return NVA_ERR_UNSUPPORTED_GEOMETRY;
    if (n_tokens == 0) return NVA_OK;
    if (!q || !k_cache || !v_cache || !block_tables || !seq_lens || !out || (bias_slope == nullptr) != (bias_rate == nullptr)) return NVA_ERR_NULL_POINTER;
    const bool decode = cu_seqlens_q == nullptr;
    if (!decode && (!token_seq || n_seqs == 0)) return NVA_ERR_NULL_POINTER;
    if (decode && n_seqs != n_tokens) return NVA_ERR_BAD_SHAPE;
    if (q_row_stride < static_cast<int64_t>(num_heads) * qk_dim || bt_row_stride < max_blocks || (gate && gate_row_stride < num_heads)) return NVA_ERR_BAD_STRIDE;
    if (static_cast<int64_t>(n_tokens) * num_heads / 4 > 0x7ffffff0LL) return NVA_ERR_BAD_SHAPE;
    ChunkAttnArgs a{};
    a.q = q; a.q_stride = q_row_stride; a.k_cache = k_cache; a.v_cache = v_cache; a.block_tables = block_tables;
    a.bt_stride = bt_row_stride; a.cu = cu_seqlens_q; a.klen = seq_lens; a.token_seq = token_seq; a.out = out;
    a.n = n_tokens; a.n_seqs = n_seqs; a.heads = num_heads; a.kv_heads = num_kv_heads; a.dim = qk_dim; a.vdim = v_dim;
    a.block_shift = shift; a.num_blocks = num_blocks; a.max_blocks = max_blocks; a.span = span;
    a.window = mask == NVA_MASK_WINDOW; a.scale = scale; a.cap = softcap; a.sinks = sinks; a.slope = bias_slope; a.rate = bias_rate; a.gate = gate; a.gate_stride = gate_row_stride;
    hipStream_t s = static_cast<hipStream_t>(stream);
    if (dtype == NVA_DTYPE_BF16 && matrix_ok(a)) {
        SplitArgs sp{};
        if (decode) {
            sp = plan_splits(num_heads, num_kv_heads, max_blocks, block_size, span);
            sp.partials = static_cast<float *>(workspace);
            if (sp.splits > 1) {
                if (!workspace) return NVA_ERR_NULL_POINTER;
                if (!aligned16(workspace)) return NVA_ERR_MISALIGNED;
                if (workspace_bytes < nva_chunk_attn_workspace_bytes(n_tokens, num_heads, num_kv_heads, v_dim, max_blocks, block_size, span))
                    return NVA_ERR_WORKSPACE_TOO_SMALL;
            }
        }
        if (std::max(qk_dim, v_dim) > 64 && std::max(qk_dim, v_dim) <= 96) return launch_matrix<96, 96>(a, sp, max_seqlen_q, s);
        if (qk_dim <= 64) return launch_matrix_dk<64>(a, sp, max_seqlen_q, s);
        if (qk_dim <= 128) return launch_matrix_dk<128>(a, sp, max_seqlen_q, s);
        return launch_matrix_dk<256>(a, sp, max_seqlen_q, s);
    }
    return dtype == NVA_DTYPE_BF16 ? launch_any<bf16_t>(a, s) : launch_any<float>(a, s);
}

extern "C" int nva_chunk_attn(const void *q, int64_t q_row_stride, const void *k_cache, const void *v_cache,
                              const int32_t *block_tables, int64_t bt_row_stride, int32_t max_blocks,
                              const int32_t *cu_seqlens_q, const int32_t *seq_lens, const int32_t *token_seq, void *out,
                              void *workspace, size_t workspace_bytes, int32_t n_tokens, int32_t n_seqs, int32_t max_seqlen_q, int32_t num_heads,
                              int32_t num_kv_heads, int32_t qk_dim, int32_t v_dim, int32_t block_size,
                              int32_t num_blocks, int32_t chunk, float scale, float softcap, int32_t dtype,
                              void *stream) {
    return nva_masked_attn(q, q_row_stride, k_cache, v_cache, block_tables, bt_row_stride, max_blocks, cu_seqlens_q, seq_lens, token_seq, out,
                           workspace, workspace_bytes, n_tokens, n_seqs, max_seqlen_q, num_heads, num_kv_heads, qk_dim, v_dim, block_size,
                           num_blocks, NVA_MASK_CHUNKS, chunk, scale, softcap, nullptr, nullptr, nullptr, nullptr, 0, dtype, stream);
}
