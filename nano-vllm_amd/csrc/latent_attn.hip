// Latent attention: a token leaves one normed latent c (rank R) and one rotated key part (rot elements), shared
// by all heads, in the paged cache.  Head h's key is [W_uk,h c | rotated part], its value W_uv,h c; the query at
// position p sees the keys (p - window, p].  Scores, weights and sums are fp32; a head may have a
// sink, one more score that belongs to no key and only enters the sum of the weights, and its result may be multiplied
// by the sigmoid of a gate projection.  Two forms:
//   absorbed   the query goes through W_uk,h^T first and meets the latents as they lie in the cache; the result
//              is a weighted latent, which goes through W_uv,h afterwards (single tokens, short portions)
//   expanded   the visible latents are gathered and multiplied out into keys and values (longer portions)
#include "nva_elem.h"
#include "nva_matrix.h"

#include <math.h>

#include <algorithm>
#include <type_traits>

namespace nva {

// where a row of a step stands: its sequence and position (-1: padded row)
struct RowsOf {
    const int32_t *cu;               // portions: [n_seqs + 1] row bounds; single tokens: null, row i is sequence i
    const int32_t *klen;             // tokens of every sequence, this step's included
    const int32_t *token_seq;        // portions: sequence of every row
    int32_t n, n_seqs;
};
__device__ __forceinline__ void place_of(const RowsOf &w, int64_t t, int &seq, int &pos) {
    if (w.cu == nullptr) {
        seq = static_cast<int>(t);
        pos = w.klen[seq] - 1;
    } else {
        seq = min(max(w.token_seq[t], 0), w.n_seqs - 1);
        pos = w.klen[seq] - (w.cu[seq + 1] - static_cast<int>(t));
    }
}

// what a head's sum of weights 2^(exponent - top) gets for its sink, and what its result is multiplied by
__device__ __forceinline__ float latent_sink(const float *sinks, int head, float top) {
    return sinks == nullptr ? 0.f : __builtin_amdgcn_exp2f(fmaf(sinks[head], 1.4426950408889634f, -top));
}
template <typename T>
__device__ __forceinline__ float latent_gate(const void *gate, int64_t stride, int64_t row, int head) {
    return gate == nullptr ? 1.0f : sigmoid_of<T>(Elem<T>::to_f32(static_cast<const T *>(gate)[row * stride + head]));
}

// V elements at e (a multiple of V, V even) of a vector whose neighbours (2i, 2i + 1) turn; table row: cos | sin
template <int V>
__device__ __forceinline__ void turn_pairs(float (&x)[V], const float *cs, int half, int e) {
#pragma unroll
    for (int i = 0; i < V; i += 2) {
        const float c = cs[(e + i) >> 1], s = cs[half + ((e + i) >> 1)];
        const float u = x[i] * c - x[i + 1] * s;
        x[i + 1] = x[i + 1] * c + x[i] * s;
        x[i] = u;
    }
}

// ---- what a token leaves behind, and its query latent ------------------------------------------------

struct LatentPrepareArgs {
    const void *x;                   // [n, q_rank + (R + rot)], row stride in elements (q_rank 0: no query latent)
    int64_t stride;
    const void *wq, *wkv;            // norm weights [q_rank], [R]
    const float *rope;               // [max_position, rot]
    void *q_out;                     // [n, q_rank] dense
    void *cache;                     // [num_slots, R + rot], or null: the layer reads another one's
    const int32_t *slot_mapping;
    int64_t num_slots;
    RowsOf rows;
    int32_t q_rank, rank, rot, max_position;
    float eps;
};

// One wavefront per row; V elements per access.
template <typename T, int V>
__global__ __launch_bounds__(256) void latent_prepare_kernel(LatentPrepareArgs a) {
    const int lane = threadIdx.x & 63;
    const int64_t t = static_cast<int64_t>(blockIdx.x) * 4 + (threadIdx.x >> 6);
    if (t >= a.rows.n) return;
    const T *x = static_cast<const T *>(a.x) + t * a.stride;
    auto normed = [&](const T *src, const T *w, int size, T *dst) __attribute__((always_inline)) {
        float sq = 0.f, v[V], g[V];
        for (int e = lane * V; e < size; e += 64 * V) {
            load_f32<T, V>(src + e, v);
#pragma unroll
            for (int i = 0; i < V; ++i) sq = fmaf(v[i], v[i], sq);
        }
        const float rstd = rsqrtf(wave_sum(sq) / static_cast<float>(size) + a.eps);
        for (int e = lane * V; e < size; e += 64 * V) {
            load_f32<T, V>(src + e, v);
            load_f32<T, V>(w + e, g);
#pragma unroll
            for (int i = 0; i < V; ++i) v[i] = v[i] * rstd * g[i];
            store_f32<T, V>(dst + e, v);
        }
    };
    if (a.q_rank > 0) normed(x, static_cast<const T *>(a.wq), a.q_rank, static_cast<T *>(a.q_out) + t * a.q_rank);
    if (a.cache == nullptr) return;
    const int64_t slot = a.slot_mapping[t];
    if (slot < 0 || slot >= a.num_slots) return;
    T *row = static_cast<T *>(a.cache) + slot * (a.rank + a.rot);
    normed(x + a.q_rank, static_cast<const T *>(a.wkv), a.rank, row);
    int seq, pos;
    place_of(a.rows, t, seq, pos);
    const float *cs = a.rope + static_cast<int64_t>(min(max(pos, 0), a.max_position - 1)) * a.rot;
    constexpr int P = V > 1 ? V : 2;
    for (int e = lane * P; e < a.rot; e += 64 * P) {
        float v[P];
        if constexpr (V > 1) {
            load_f32<T, P>(x + a.q_rank + a.rank + e, v);
        } else {
            v[0] = Elem<T>::to_f32(x[a.q_rank + a.rank + e]);
            v[1] = Elem<T>::to_f32(x[a.q_rank + a.rank + e + 1]);
        }
        turn_pairs<P>(v, cs, a.rot / 2, e);
        if constexpr (V > 1) {
            store_f32<T, P>(row + a.rank + e, v);
        } else {
            row[a.rank + e] = Elem<T>::from_f32(v[0]);
            row[a.rank + e + 1] = Elem<T>::from_f32(v[1]);
        }
    }
}

// ---- absorbed form ------------------------------------------------------------------------------------

struct LatentAttnArgs {
    const void *q_lat;               // [n, H, R] dense
    const void *q_rot;               // [n, H, rot]: not yet rotated; strides in elements
    int64_t qr_row, qr_head;
    const void *gate;                // [n, H] logits, row stride in elements, or null
    int64_t gate_stride;
    const float *sinks;              // [H] or null
    const float *rope;
    const void *cache;               // [num_blocks, block, R + rot]
    const int32_t *block_tables;     // [n_seqs, >= max_blocks]
    int64_t bt_stride;
    void *out;                       // [n, H, R] dense
    RowsOf rows;
    int32_t heads, rank, rot, block_shift, num_blocks, max_blocks, window, max_position;
    float scale;
};

// One wavefront per (row, head), any sizes, bf16 or fp32: lanes are keys for the scores and latent
// elements for the weighted sum; running maximum and sum per block of 64 keys.
constexpr int kLatentMax = 1024;

template <typename T>
__global__ __launch_bounds__(256) void latent_attn_any_kernel(LatentAttnArgs a) {
    __shared__ float sh_q[4][kLatentMax];
    const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
    const int64_t item = static_cast<int64_t>(blockIdx.x) * 4 + wave;
    const bool live = item < static_cast<int64_t>(a.rows.n) * a.heads;
    const int64_t t = live ? item / a.heads : 0;
    const int head = live ? static_cast<int>(item % a.heads) : 0;
    const int width = a.rank + a.rot;
    int seq, pos;
    place_of(a.rows, t, seq, pos);
    if (live) {
        const T *q = static_cast<const T *>(a.q_lat) + item * a.rank;
        for (int i = lane; i < a.rank; i += 64) sh_q[wave][i] = Elem<T>::to_f32(q[i]);
        const T *qr = static_cast<const T *>(a.q_rot) + t * a.qr_row + head * a.qr_head;
        const float *cs = a.rope + static_cast<int64_t>(min(max(pos, 0), a.max_position - 1)) * a.rot;
        for (int e = 2 * lane; e < a.rot; e += 128) {
            float v[2] = {Elem<T>::to_f32(qr[e]), Elem<T>::to_f32(qr[e + 1])};
            turn_pairs<2>(v, cs, a.rot / 2, e);
            sh_q[wave][a.rank + e] = v[0];
            sh_q[wave][a.rank + e + 1] = v[1];
        }
    }
    __syncthreads();
    if (!live) return;
    float m = -INFINITY, sum = 0.f;
    float acc[kLatentMax / 64];
#pragma unroll
    for (int i = 0; i < kLatentMax / 64; ++i) acc[i] = 0.f;
    const int bmask = (1 << a.block_shift) - 1;
    for (int j0 = max(0, pos - a.window + 1); j0 <= pos; j0 += 64) {
        const int j = j0 + lane;
        int64_t row = -1;                                  // cache row of this lane's key
        if (j <= pos && (j >> a.block_shift) < a.max_blocks) {
            const int blk = a.block_tables[seq * a.bt_stride + (j >> a.block_shift)];
            if (static_cast<uint32_t>(blk) < static_cast<uint32_t>(a.num_blocks))
                row = (static_cast<int64_t>(blk) << a.block_shift) + (j & bmask);
        }
        float s = -INFINITY;
        if (row >= 0) {
            const T *k = static_cast<const T *>(a.cache) + row * width;
            float d = 0.f;
            for (int i = 0; i < width; ++i) d = fmaf(sh_q[wave][i], Elem<T>::to_f32(k[i]), d);
            s = d * a.scale;
        }
        const float m_new = fmaxf(m, wave_max(s));
        if (m_new == -INFINITY) continue;
        const float p = row >= 0 ? exp_of<T>(s - m_new) : 0.f;
        const float keep = m == -INFINITY ? 0.f : exp_of<T>(m - m_new);
        sum = sum * keep + wave_sum(p);
        m = m_new;
#pragma unroll
        for (int i = 0; i < kLatentMax / 64; ++i) acc[i] *= keep;
        const int count = min(64, pos - j0 + 1);
        for (int jj = 0; jj < count; ++jj) {
            const int64_t vrow = __shfl(row, jj, 64);
            if (vrow < 0) continue;
            const float w = __shfl(p, jj, 64);
            const T *v = static_cast<const T *>(a.cache) + vrow * width;
#pragma unroll
            for (int i = 0; i < kLatentMax / 64; ++i)
                if (i * 64 + lane < a.rank) acc[i] = fmaf(w, Elem<T>::to_f32(v[i * 64 + lane]), acc[i]);
        }
    }
    T *out = static_cast<T *>(a.out) + item * a.rank;
    if (a.sinks != nullptr && sum > 0.f) sum += exp_of<T>(a.sinks[head] - m);
    const float f = sum > 0.f ? latent_gate<T>(a.gate, a.gate_stride, t, head) / sum : 0.f;
#pragma unroll
    for (int i = 0; i < kLatentMax / 64; ++i)
        if (i * 64 + lane < a.rank) out[i * 64 + lane] = Elem<T>::from_f32(acc[i] * f);
}

// bf16 on the matrix cores (v_mfma_f32_16x16x32_bf16, transposed: S^T = K Q^T, O^T += C^T P^T).  A workgroup takes
// one (row, range of keys, 16 NH heads) and walks the range in tiles of 64 keys.  Wavefront w loads 16 of them from memory
// straight into operand registers, forms their scores, and puts the latents into LDS, where every wavefront reads
// its quarter of the latent columns through the transpose.  The score accumulators (register i of lane l: key 4 (l / 16) + i)
// are a legal key order for the second product, so the weights go to the other wavefronts lane by lane; fp32, they
// enter it as the sum of two bf16 numbers.  The next tile's loads go out as soon as the registers are free.  The
// reference of the weights is shared by the wavefronts and moves only when a score passes it by more than 2^8.  With
// more than one range per row the results are partial (fp32 sums, sum of the weights, reference exponent)
// and latent_merge_kernel adds them up.  kExact: the model's sizes are those the registers are laid out for.
struct LatentSplit {
    float *partials;         // [n, splits, heads, R + 4]: sums, sum of the weights, reference exponent
    int32_t splits, keys;    // ranges per row, keys per range (a multiple of 64)
    int32_t head_groups;     // groups of 16 NH heads
};
constexpr int kRowTile = 64;

template <int RK, int DR, int NH, bool kExact>
__global__ __launch_bounds__(256, 2) void latent_rows_kernel(const LatentAttnArgs a, const LatentSplit sp) {
    constexpr int kKS = RK / 32, kAll = (RK + DR) / 32, kPitch = RK * 2 + 32;
    constexpr int kDB = RK / 64;                         // value blocks of 16 columns per wavefront
    __shared__ __attribute__((aligned(16))) unsigned char smem[kRowTile * kPitch];
    __shared__ u32x4_t sh_p[NH][4][64];
    __shared__ float sh_m[NH][4][16], sh_l[NH][4][16];
    const int tid = threadIdx.x, lane = tid & 63;
    const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
    const int r = lane & 15, g = lane >> 4;
    // (row, range) pairs are dealt out over the XCDs, a pair's head groups to the same one; rows are the fastest
    // index, so that ranges past the end of short sequences spread over the CUs
    const int hg = blockIdx.x / 8 % sp.head_groups;
    const int64_t item = static_cast<int64_t>(blockIdx.x) / (8 * sp.head_groups) * 8 + blockIdx.x % 8;
    if (item >= static_cast<int64_t>(a.rows.n) * sp.splits) return;
    const int64_t t = item % a.rows.n;
    const int split = static_cast<int>(item / a.rows.n), head0 = hg * 16 * NH;
    const int nheads = min(16 * NH, a.heads - head0);
    int seq, pos;
    place_of(a.rows, t, seq, pos);
    bf16_t *out = static_cast<bf16_t *>(a.out) + (t * a.heads + head0) * a.rank;
    if (pos < 0) {
        if (sp.splits == 1)
            for (int i = tid; i < nheads * a.rank; i += 256) out[i] = 0;
        return;
    }
    const int lo = max(0, pos - a.window + 1), first = (lo & ~(kRowTile - 1)) + split * sp.keys;
    const int last = min(pos, first + sp.keys - 1);      // last key of this range
    if (first > last) return;
    const int ntiles = (last - first) / kRowTile + 1, width = a.rank + a.rot;
    const int bmask = (1 << a.block_shift) - 1;
    const lds_char_ptr lds = (lds_char_ptr)(&smem[0]);
    const bf16_t *cache = static_cast<const bf16_t *>(a.cache);

    auto block_of = [&](int tile) __attribute__((always_inline)) -> int {
        const int col = (first + tile * kRowTile) >> a.block_shift;
        return tile < ntiles && col < a.max_blocks ? a.block_tables[seq * a.bt_stride + col] : -1;
    };
    u32x4_t kf[kAll];
    auto fetch = [&](int tile, int blk) __attribute__((always_inline)) {
        const int key0 = first + tile * kRowTile;
        const bool ok = static_cast<uint32_t>(blk) < static_cast<uint32_t>(a.num_blocks);
        if (!ok) return;
        const int row = min(16 * wave + r, last - key0);             // rows past the last key repeat it and are masked
        const bf16_t *base = cache + ((static_cast<int64_t>(blk) << a.block_shift) + (key0 & bmask) + row) * width + 8 * g;
#pragma unroll
        for (int ks = 0; ks < kAll; ++ks) {
            const int e = ks < kKS ? 32 * ks : 32 * (ks - kKS);
            const bool in = kExact || e + 8 * g < (ks < kKS ? a.rank : a.rot);
            if (!kExact) kf[ks] = u32x4_t{0, 0, 0, 0};
            if (in) kf[ks] = *reinterpret_cast<const u32x4_t *>(base + (ks < kKS ? e : a.rank + e));
        }
    };
    int blk = block_of(0), blk_next = block_of(1);
    fetch(0, blk);
    u32x4_t qf[NH][kAll];
    {
        const float *cs = a.rope + static_cast<int64_t>(min(pos, a.max_position - 1)) * a.rot;
#pragma unroll
        for (int h = 0; h < NH; ++h) {
            const int head = head0 + min(16 * h + r, nheads - 1);
            const bf16_t *ql = static_cast<const bf16_t *>(a.q_lat) + (t * a.heads + head) * a.rank;
            const bf16_t *qr = static_cast<const bf16_t *>(a.q_rot) + t * a.qr_row + head * a.qr_head;
#pragma unroll
            for (int ks = 0; ks < kAll; ++ks) {
                qf[h][ks] = u32x4_t{0, 0, 0, 0};
                if (ks < kKS) {
                    const int e = 32 * ks + 8 * g;
                    if (kExact || e < a.rank) qf[h][ks] = *reinterpret_cast<const u32x4_t *>(ql + e);
                } else {
                    const int e = 32 * (ks - kKS) + 8 * g;
                    if (kExact || e < a.rot) {
                        float v[8];
                        load_f32<bf16_t, 8>(qr + e, v);
                        turn_pairs<8>(v, cs, a.rot / 2, e);
#pragma unroll
                        for (int i = 0; i < 4; ++i) qf[h][ks][i] = pack_bf16x2(v[2 * i], v[2 * i + 1]);
                    }
                }
            }
        }
    }
    f32x4_t oacc[NH][kDB];
    float lsum[NH], m[NH];
#pragma unroll
    for (int h = 0; h < NH; ++h) {
        lsum[h] = 0.f;
        m[h] = -INFINITY;
#pragma unroll
        for (int db = 0; db < kDB; ++db) oacc[h][db] = f32x4_t{0.f, 0.f, 0.f, 0.f};
    }
    const float to_exp2 = a.scale * 1.4426950408889634f;
    const lds_char_ptr vw = lds + (16 * wave + r) * kPitch + 16 * g;
    const lds_char_ptr vl = lds + (4 * g + (r >> 2)) * kPitch + 8 * (r & 3) + wave * (RK / 4) * 2;
    for (int tile = 0; tile < ntiles; ++tile) {
        const int key0 = first + tile * kRowTile;
        const bool ok = static_cast<uint32_t>(blk) < static_cast<uint32_t>(a.num_blocks);
        const int blk_this = blk_next;
        if (!ok) {                                       // (the whole workgroup skips it)
            blk = blk_this;
            blk_next = block_of(tile + 2);
            if (tile + 1 < ntiles) fetch(tile + 1, blk);
            continue;
        }
        f32x4_t s[NH][2];                                // two chains, added below
        float x[NH][4];
#pragma unroll
        for (int h = 0; h < NH; ++h) s[h][0] = s[h][1] = f32x4_t{0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int ks = 0; ks < kAll; ++ks)
#pragma unroll
            for (int h = 0; h < NH; ++h) s[h][ks & 1] = mfma16(kf[ks], qf[h][ks], s[h][ks & 1]);
        const int key = key0 + 16 * wave + 4 * g;
#pragma unroll
        for (int h = 0; h < NH; ++h) {
            float mx = -INFINITY;
#pragma unroll
            for (int i = 0; i < 4; ++i) {
                x[h][i] = key + i >= lo && key + i <= last ? (s[h][0][i] + s[h][1][i]) * to_exp2 : -INFINITY;
                mx = fmaxf(mx, x[h][i]);
            }
            mx = fmaxf(mx, __shfl_xor(mx, 16, 64));
            mx = fmaxf(mx, __shfl_xor(mx, 32, 64));
            if (g == 0) sh_m[h][wave][r] = mx;
        }
        __syncthreads();                                 // maxima are there; the tile before has been read
#pragma unroll
        for (int ks = 0; ks < kKS; ++ks) *(lds_u32x4_ptr)(vw + 64 * ks) = kf[ks];
        blk = blk_this;
        blk_next = block_of(tile + 2);
        if (tile + 1 < ntiles) fetch(tile + 1, blk);
#pragma unroll
        for (int h = 0; h < NH; ++h) {
            const float mx = fmaxf(fmaxf(sh_m[h][0][r], sh_m[h][1][r]), fmaxf(sh_m[h][2][r], sh_m[h][3][r]));
            if (__any(mx > m[h] + 8.0f)) {               // (the same in every wavefront)
                const float m_new = fmaxf(m[h], mx);
                const float keep = m[h] == -INFINITY ? 0.f : __builtin_amdgcn_exp2f(m[h] - m_new);
                m[h] = m_new;
                lsum[h] *= keep;
#pragma unroll
                for (int db = 0; db < kDB; ++db)
#pragma unroll
                    for (int i = 0; i < 4; ++i) oacc[h][db][i] *= keep;
            }
            const float ref = m[h] == -INFINITY ? 0.f : m[h];
            float p[4];
#pragma unroll
            for (int i = 0; i < 4; ++i) {
                p[i] = __builtin_amdgcn_exp2f(x[h][i] - ref);
                lsum[h] += p[i];
            }
            uint32_t h0, l0, h1, l1;
            split_pair(p[0], p[1], h0, l0);
            split_pair(p[2], p[3], h1, l1);
            sh_p[h][wave][lane] = u32x4_t{h0, h1, l0, l1};
        }
        __syncthreads();
#pragma unroll
        for (int st = 0; st < 2; ++st) {
            u32x4_t ph[NH], pl[NH];
#pragma unroll
            for (int h = 0; h < NH; ++h) {
                const u32x4_t p0 = sh_p[h][2 * st][lane], p1 = sh_p[h][2 * st + 1][lane];
                ph[h] = u32x4_t{p0[0], p0[1], p1[0], p1[1]};
                pl[h] = u32x4_t{p0[2], p0[3], p1[2], p1[3]};
            }
#pragma unroll
            for (int db = 0; db < kDB; ++db) {
                const s16x4_t v0 = __builtin_amdgcn_ds_read_tr16_b64_v4i16((lds_s16x4_ptr)(vl + 32 * st * kPitch + 32 * db));
                const s16x4_t v1 = __builtin_amdgcn_ds_read_tr16_b64_v4i16((lds_s16x4_ptr)(vl + (32 * st + 16) * kPitch + 32 * db));
                const u32x4_t vf = __builtin_bit_cast(u32x4_t, __builtin_shufflevector(v0, v1, 0, 1, 2, 3, 4, 5, 6, 7));
#pragma unroll
                for (int h = 0; h < NH; ++h) {
                    oacc[h][db] = mfma16(vf, ph[h], oacc[h][db]);
                    oacc[h][db] = mfma16(vf, pl[h], oacc[h][db]);
                }
            }
        }
    }
    // sums of the weights: a wavefront's keys are spread over its lane groups, the tile's over the wavefronts
#pragma unroll
    for (int h = 0; h < NH; ++h) {
        lsum[h] += __shfl_xor(lsum[h], 16, 64);
        lsum[h] += __shfl_xor(lsum[h], 32, 64);
        if (g == 0) sh_l[h][wave][r] = lsum[h];
    }
    __syncthreads();
#pragma unroll
    for (int h = 0; h < NH; ++h) {
        const int hh = 16 * h + r;
        if (hh >= nheads) continue;
        const float l = (sh_l[h][0][r] + sh_l[h][1][r]) + (sh_l[h][2][r] + sh_l[h][3][r]);
        if (sp.splits == 1) {
            const float f = l > 0.f ? latent_gate<bf16_t>(a.gate, a.gate_stride, t, head0 + hh) / (l + latent_sink(a.sinks, head0 + hh, m[h])) : 0.f;
#pragma unroll
            for (int db = 0; db < kDB; ++db) {
                const int c = wave * (RK / 4) + 16 * db + 4 * g;
                if (kExact || c < a.rank)
                    *reinterpret_cast<u32x2_t *>(out + hh * a.rank + c) = u32x2_t{pack_bf16x2(oacc[h][db][0] * f, oacc[h][db][1] * f), pack_bf16x2(oacc[h][db][2] * f, oacc[h][db][3] * f)};
            }
        } else {
            float *part = sp.partials + ((t * sp.splits + split) * a.heads + head0 + hh) * (a.rank + 4);
#pragma unroll
            for (int db = 0; db < kDB; ++db) {
                const int c = wave * (RK / 4) + 16 * db + 4 * g;
                if (kExact || c < a.rank) *reinterpret_cast<f32x4_t *>(part + c) = oacc[h][db];
            }
            if (wave == 0 && g == 0) { part[a.rank] = l; part[a.rank + 1] = m[h]; }
        }
    }
}

// Adds the partial results of the ranges that hold keys (at most 64): one wavefront per 256 columns of a (row,
// head), several ranges' loads in flight together.
__global__ __launch_bounds__(256) void latent_merge_kernel(const LatentAttnArgs a, const LatentSplit sp, const int32_t pieces) {
    const int lane = threadIdx.x & 63;
    const int64_t job = static_cast<int64_t>(blockIdx.x) * 4 + (threadIdx.x >> 6);
    const int64_t item = job / pieces;
    if (item >= static_cast<int64_t>(a.rows.n) * a.heads) return;
    const int c = static_cast<int>(job % pieces) * 256 + 4 * lane;
    const int64_t t = item / a.heads;
    const int head = static_cast<int>(item % a.heads);
    int seq, pos;
    place_of(a.rows, t, seq, pos);
    const int first = max(0, pos - a.window + 1) & ~(kRowTile - 1);
    const int count = pos < 0 ? 0 : min(sp.splits, (pos - first) / sp.keys + 1);
    const int pitch = a.rank + 4;
    const float *part = sp.partials + (t * sp.splits * a.heads + head) * pitch;
    const int64_t step = static_cast<int64_t>(a.heads) * pitch;
    // lane j holds sum and reference of range j
    const float my_l = lane < count ? part[lane * step + a.rank] : 0.f;
    const float my_m = lane < count ? part[lane * step + a.rank + 1] : -INFINITY;
    const float gate = latent_gate<bf16_t>(a.gate, a.gate_stride, t, head);
    constexpr int kAhead = 8;
    f32x4_t p[kAhead], o = {0.f, 0.f, 0.f, 0.f};
    const bool in = c < a.rank;                          // (the rank is a multiple of 8)
    auto fetch = [&](int j0) __attribute__((always_inline)) {
#pragma unroll
        for (int j = 0; j < kAhead; ++j)
            if (in && j0 + j < count) p[j] = *reinterpret_cast<const f32x4_t *>(part + (j0 + j) * step + c);
    };
    fetch(0);
    const float top = wave_max(my_m);
    const float f = my_m == -INFINITY ? 0.f : __builtin_amdgcn_exp2f(my_m - top);
    const float l = wave_sum(my_l * f);
    const float inv = l > 0.f ? gate / (l + latent_sink(a.sinks, head, top)) : 0.f;
    for (int j0 = 0; j0 < count; j0 += kAhead) {
#pragma unroll
        for (int j = 0; j < kAhead; ++j) {
            const float w = __shfl(f, min(j0 + j, 63), 64);
            if (j0 + j < count)
#pragma unroll
                for (int i = 0; i < 4; ++i) o[i] = fmaf(p[j][i], w, o[i]);
        }
        if (j0 + kAhead < count) fetch(j0 + kAhead);
    }
    if (in)
        *reinterpret_cast<u32x2_t *>(static_cast<bf16_t *>(a.out) + item * a.rank + c) = u32x2_t{pack_bf16x2(o[0] * inv, o[1] * inv), pack_bf16x2(o[2] * inv, o[3] * inv)};
}

// How the keys of a row are split.  Depends on shapes only.
static LatentSplit plan_latent(int32_t rows, int32_t heads, int32_t rank, int32_t max_blocks, int32_t block_size, int32_t window) {
    LatentSplit sp{};
    const int nh = heads > 16 && rank <= 256 ? 2 : 1;    // (two groups' registers do not fit beside a longer latent)
    sp.head_groups = (heads + 16 * nh - 1) / (16 * nh);
    const int64_t most = std::min(static_cast<int64_t>(window), static_cast<int64_t>(max_blocks) * block_size) + kRowTile - 1;   // keys one row can see, from a tile's start on
    const int64_t want = std::max<int64_t>(1, 1024 / std::max<int64_t>(1, static_cast<int64_t>(rows) * sp.head_groups));
    const int64_t least = static_cast<int64_t>(rows) * sp.head_groups <= 32 ? 128 : 256;
    int64_t keys = std::max({least, (most + want - 1) / want, (most + 63) / 64});
    keys = (keys + kRowTile - 1) / kRowTile * kRowTile;
    sp.keys = static_cast<int32_t>(keys);
    sp.splits = static_cast<int32_t>(std::max(static_cast<int64_t>(1), (most + keys - 1) / keys));
    return sp;
}

template <int RK, int DR, int NH, bool kExact>
static int launch_latent_rows(const LatentAttnArgs &a, const LatentSplit &sp, hipStream_t s) {
    const int64_t items = (static_cast<int64_t>(a.rows.n) * sp.splits + 7) / 8 * 8;
    if (items * sp.head_groups > 0x7fffffffLL) return NVA_ERR_BAD_SHAPE;
    const dim3 block(256);
    hipLaunchKernelGGL((latent_rows_kernel<RK, DR, NH, kExact>), dim3(static_cast<uint32_t>(items * sp.head_groups)), block, 0, s, a, sp);
    const int rc = launch_status();
    if (rc != NVA_OK || sp.splits == 1) return rc;
    const int32_t pieces = (a.rank + 255) / 256;
    hipLaunchKernelGGL(latent_merge_kernel, dim3(static_cast<uint32_t>((static_cast<int64_t>(a.rows.n) * a.heads * pieces + 3) / 4)), block, 0, s, a, sp, pieces);
    return launch_status();
}

static bool latent_rows_ok(int32_t rank, int32_t rot, int32_t dtype) {
    return dtype == NVA_DTYPE_BF16 && rank % 8 == 0 && rot % 8 == 0 && rank <= 512 && rot <= 64;
}

// ---- expanded form ------------------------------------------------------------------------------------

// Visible latents of every sequence, one after the other: row i of sequence s is the cache row of position
// seq_lens[s] - (key_cu[s + 1] - key_cu[s]) + i.  One wavefront per row; V elements per access.
template <typename T, int V>
__global__ __launch_bounds__(256) void latent_gather_kernel(const T *cache, const int32_t *block_tables, int64_t bt_stride, const int32_t *key_cu,
                                                            const int32_t *klen, T *out, int32_t n_keys, int32_t n_seqs, int32_t width,
                                                            int32_t block_shift, int32_t num_blocks, int32_t max_blocks) {
    const int lane = threadIdx.x & 63;
    const int row = blockIdx.x * 4 + (threadIdx.x >> 6);
    if (row >= n_keys) return;
    int lo = 0, hi = n_seqs - 1;                           // the sequence: last one that begins at or before the row
    while (lo < hi) {
        const int mid = (lo + hi + 1) >> 1;
        if (key_cu[mid] <= row) lo = mid; else hi = mid - 1;
    }
    const int pos = klen[lo] - (key_cu[lo + 1] - row);
    const int col = pos >> block_shift;
    const int blk = pos >= 0 && col < max_blocks ? block_tables[lo * bt_stride + col] : -1;
    const bool ok = static_cast<uint32_t>(blk) < static_cast<uint32_t>(num_blocks);
    const T *src = cache + ((static_cast<int64_t>(ok ? blk : 0) << block_shift) + (ok ? pos & ((1 << block_shift) - 1) : 0)) * width;
    for (int e = lane * V; e < width; e += 64 * V) {
        float v[V];
        load_f32<T, V>(src + e, v);
#pragma unroll
        for (int i = 0; i < V; ++i) v[i] = ok ? v[i] : 0.f;
        store_f32<T, V>(out + static_cast<int64_t>(row) * width + e, v);
    }
}

struct LatentPrefillArgs {
    const bf16_t *q;                 // [n, H, dim + rot]: the rotated part not yet rotated; row stride in elements
    int64_t q_stride;
    const bf16_t *kv;                // [n_keys, H dim | H vdim], row stride in elements
    int64_t kv_stride;
    const bf16_t *k_rot;             // [n_keys, rot], row stride in elements
    int64_t kr_stride;
    const bf16_t *gate;              // or null
    int64_t gate_stride;
    const float *sinks;              // [H] or null
    const float *rope;
    const int32_t *cu, *klen, *key_cu;
    bf16_t *out;                     // [n, H, vdim] dense
    int32_t heads, dim, rot, vdim, window, max_position;
    float scale;
};

// A workgroup of four wavefronts takes 4 * 16 * NQ queries of one head and walks their keys in tiles of 64,
// through LDS.  DN, DR, DV: sizes the registers are laid out for.  kDirect (the model's sizes are
// exactly these): tiles travel global -> LDS (two buffers) without a register in between, the LDS image laid out in 1 KB blocks
// of 16 keys x 32 dims with the 16-byte pieces permuted so that operand reads spread over the banks.  Otherwise
// (smaller sizes, multiples of 8) tiles go through registers into padded rows, zero-filled to DN, DR and DV.
// A running maximum is the reference of the weights; it moves only when a score passes it by more than 2^8.
template <int DN, int DR, int DV, int NQ, bool kDirect>
__global__ __launch_bounds__(256, DN + DR + DV > 384 ? 1 : 2) void latent_prefill_kernel(const LatentPrefillArgs a, const int32_t q_tiles) {
    constexpr int DK = DN + DR, kBM = 64 * NQ, kBN = 64;
    constexpr int kKPitch = DK * 2 + 16, kVPitch = DV * 2 + 32;
    constexpr int kKPieces = DK / 32, kVPieces = DV / 32;           // 16-byte pieces of a tile per thread
    constexpr int kKTile = kDirect ? kBN * DK * 2 : kBN * kKPitch, kVTile = kDirect ? kBN * DV * 2 : kBN * kVPitch;
    constexpr int kBufs = kDirect ? 2 : 1;                          // (through registers, one tile in LDS is enough)
    __shared__ __attribute__((aligned(1024))) unsigned char smem[kBufs * (kKTile + kVTile)];
    const lds_char_ptr lds = (lds_char_ptr)(&smem[0]);
    // heads fastest, query tiles last to first: the workgroups that share keys run close together on one XCD
    const int head = blockIdx.x % a.heads;
    const int rest = blockIdx.x / a.heads;
    const int row0 = (q_tiles - 1 - rest % q_tiles) * kBM;
    const int seq = rest / q_tiles;
    const int tid = threadIdx.x, lane = tid & 63;
    const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
    const int r = lane & 15, g = lane >> 4;
    const int t0 = a.cu[seq], lq = a.cu[seq + 1] - t0;
    if (row0 >= lq) return;
    const int klen = a.klen[seq], start = klen - lq;
    if (start < 0) return;
    const int last_row = min(row0 + kBM, lq) - 1;
    const int key_end = start + last_row;                            // last key any query of the tile sees
    const int key_base = klen - (a.key_cu[seq + 1] - a.key_cu[seq]); // position of the sequence's first gathered key
    const int key_begin = max(max(0, start + row0 - a.window + 1), key_base);
    if (key_begin > key_end) return;
    const int ntiles = (key_end - key_begin) / kBN + 1;
    const int64_t row_base = a.key_cu[seq] - key_base;               // gathered row of position 0
    const bf16_t *kc = a.kv + static_cast<int64_t>(head) * a.dim;
    const bf16_t *vc = a.kv + static_cast<int64_t>(a.heads) * a.dim + static_cast<int64_t>(head) * a.vdim;

    // queries of this wavefront, rotated on the way
    int pos[NQ], lo[NQ];
    u32x4_t qf[NQ][DK / 32];
#pragma unroll
    for (int qa = 0; qa < NQ; ++qa) {
        const int row = row0 + wave * 16 * NQ + 16 * qa + r;
        pos[qa] = start + row;
        lo[qa] = max(0, pos[qa] - a.window + 1);
        const bf16_t *q = a.q + static_cast<int64_t>(t0 + min(row, lq - 1)) * a.q_stride + static_cast<int64_t>(head) * (a.dim + a.rot);
        const float *cs = a.rope + static_cast<int64_t>(min(pos[qa], a.max_position - 1)) * a.rot;
#pragma unroll
        for (int ks = 0; ks < DK / 32; ++ks) {
            qf[qa][ks] = u32x4_t{0, 0, 0, 0};
            if (ks < DN / 32) {
                const int e = 32 * ks + 8 * g;
                if (e < a.dim) qf[qa][ks] = *reinterpret_cast<const u32x4_t *>(q + e);
            } else {
                const int e = 32 * (ks - DN / 32) + 8 * g;
                if (e < a.rot) {
                    float v[8];
                    load_f32<bf16_t, 8>(q + a.dim + e, v);
                    turn_pairs<8>(v, cs, a.rot / 2, e);
#pragma unroll
                    for (int i = 0; i < 4; ++i) qf[qa][ks][i] = pack_bf16x2(v[2 * i], v[2 * i + 1]);
                }
            }
        }
    }
    const int w_first = start + row0 + wave * 16 * NQ;               // the wavefront's queries: first and last position
    const int w_last = min(w_first + 16 * NQ - 1, key_end);
    const bool w_live = row0 + wave * 16 * NQ < lq;
    const int w_lo = max(0, w_first - a.window + 1);                 // oldest key one of them sees
    const int w_lo_all = max(0, w_last - a.window + 1);              // keys from here to w_first are seen by all

    u32x4_t kreg[kDirect ? 1 : kKPieces], vreg[kDirect ? 1 : kVPieces];
    const int lk16 = lane >> 2, lj = lane & 3;
    const uint32_t lds_k0 = __builtin_amdgcn_readfirstlane(static_cast<uint32_t>(reinterpret_cast<uintptr_t>(lds)) + wave * (DK / 32) * 1024);
    const uint32_t lds_v0 = __builtin_amdgcn_readfirstlane(static_cast<uint32_t>(reinterpret_cast<uintptr_t>(lds)) + kBufs * kKTile + wave * (DV / 32) * 1024);
    uint32_t koff = 0, roff = 0, voff = 0;
    auto fetch = [&](int tile, int buf) __attribute__((always_inline)) {
        const int key0 = key_begin + tile * kBN;
        const int64_t base = row_base + key0;
        if constexpr (kDirect) {
            const int row = min(wave * 16 + lk16, key_end - key0);   // rows past the last key repeat it and are masked
            const int kpiece = (lj ^ ((0 - (lk16 >> 2)) & 3)) * 8;
            koff = static_cast<uint32_t>(row * a.kv_stride + kpiece) * 2;
            roff = static_cast<uint32_t>(row * a.kr_stride + kpiece) * 2;
            voff = static_cast<uint32_t>(row * a.kv_stride + (lj ^ (2 * ((lk16 >> 2) & 1))) * 8) * 2;
            const char *kb = reinterpret_cast<const char *>(kc + base * a.kv_stride), *vb = reinterpret_cast<const char *>(vc + base * a.kv_stride);
            const char *rb = reinterpret_cast<const char *>(a.k_rot + base * a.kr_stride);
#pragma unroll
            for (int x = 0; x < DN / 32; ++x) load_to_lds_16(kb + 64 * x, koff, lds_k0 + buf * kKTile + 1024 * x);
#pragma unroll
            for (int x = 0; x < DR / 32; ++x) load_to_lds_16(rb + 64 * x, roff, lds_k0 + buf * kKTile + 1024 * (DN / 32 + x));
#pragma unroll
            for (int x = 0; x < DV / 32; ++x) load_to_lds_16(vb + 64 * x, voff, lds_v0 + buf * kVTile + 1024 * x);
        } else {
#pragma unroll
            for (int i = 0; i < kKPieces; ++i) {
                const int p = i * 256 + tid, row = p / (DK / 8), c = p % (DK / 8) * 8;
                kreg[i] = u32x4_t{0, 0, 0, 0};
                if (key0 + row <= key_end) {
                    if (c < DN) { if (c < a.dim) kreg[i] = *reinterpret_cast<const u32x4_t *>(kc + (base + row) * a.kv_stride + c); }
                    else if (c - DN < a.rot) kreg[i] = *reinterpret_cast<const u32x4_t *>(a.k_rot + (base + row) * a.kr_stride + (c - DN));
                }
            }
#pragma unroll
            for (int i = 0; i < kVPieces; ++i) {
                const int p = i * 256 + tid, row = p / (DV / 8), e = p % (DV / 8) * 8;
                vreg[i] = u32x4_t{0, 0, 0, 0};
                if (key0 + row <= key_end && e < a.vdim) vreg[i] = *reinterpret_cast<const u32x4_t *>(vc + (base + row) * a.kv_stride + e);
            }
        }
    };
    auto put = [&](int buf) __attribute__((always_inline)) {
        if constexpr (kDirect) {
            loads_issued(koff, voff);
            loads_issued(roff, roff);
            asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
        } else {
            const lds_char_ptr kl = lds + buf * kKTile, vl = lds + kBufs * kKTile + buf * kVTile;
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
    float lsum[NQ], m[NQ];
#pragma unroll
    for (int qa = 0; qa < NQ; ++qa) {
        lsum[qa] = 0.f;
        m[qa] = -INFINITY;
#pragma unroll
        for (int db = 0; db < DV / 16; ++db) oacc[db][qa] = f32x4_t{0.f, 0.f, 0.f, 0.f};
    }
    const float to_exp2 = a.scale * 1.4426950408889634f;

    auto attend = [&](auto masked_c, int key0, int buf) __attribute__((always_inline)) {
        constexpr bool kMasked = decltype(masked_c)::value;
        const lds_char_ptr kl = lds + buf * kKTile + (kDirect ? 16 * (4 * r + (g ^ ((0 - (r >> 2)) & 3))) : r * kKPitch + 16 * g);
        const lds_char_ptr vl = lds + kBufs * kKTile + buf * kVTile + (4 * g + (r >> 2)) * (kDirect ? 64 : kVPitch) + 8 * (r & 3);
        auto kpiece = [&](int kb, int ks) __attribute__((always_inline)) -> u32x4_t {
            return *(lds_u32x4_ptr)(kl + (kDirect ? (kb * (DK / 32) + ks) * 1024 : kb * 16 * kKPitch + ks * 64));
        };
        auto vpiece = [&](int kb, int db) __attribute__((always_inline)) -> s16x4_t {
            return __builtin_amdgcn_ds_read_tr16_b64_v4i16((lds_s16x4_ptr)(
                vl + (kDirect ? (kb * (DV / 32) + (db >> 1)) * 1024 + 32 * ((g ^ db) & 1) : kb * 16 * kVPitch + 32 * db)));
        };
        f32x4_t sacc[4][NQ];
#pragma unroll
        for (int kb = 0; kb < 4; ++kb) {
#pragma unroll
            for (int qa = 0; qa < NQ; ++qa) sacc[kb][qa] = f32x4_t{0.f, 0.f, 0.f, 0.f};
#pragma unroll
            for (int ks = 0; ks < DK / 32; ++ks) {
                const u32x4_t kf = kpiece(kb, ks);
#pragma unroll
                for (int qa = 0; qa < NQ; ++qa) sacc[kb][qa] = mfma16(kf, qf[qa][ks], sacc[kb][qa]);
            }
        }
        auto seen = [&](int qa, int kb, int i) __attribute__((always_inline)) -> bool {
            const int key = key0 + 16 * kb + 4 * g + i;
            return !kMasked || (key >= lo[qa] && key <= pos[qa]);
        };
#pragma unroll
        for (int qa = 0; qa < NQ; ++qa) {
            float mx = -INFINITY;
#pragma unroll
            for (int kb = 0; kb < 4; ++kb)
#pragma unroll
                for (int i = 0; i < 4; ++i)
                    if (seen(qa, kb, i)) mx = fmaxf(mx, sacc[kb][qa][i] * to_exp2);
            mx = fmaxf(mx, __shfl_xor(mx, 16, 64));
            mx = fmaxf(mx, __shfl_xor(mx, 32, 64));
            if (__any(mx > m[qa] + 8.0f)) {
                const float m_new = fmaxf(m[qa], mx);
                const float keep = m[qa] == -INFINITY ? 0.f : __builtin_amdgcn_exp2f(m[qa] - m_new);
                m[qa] = m_new;
                lsum[qa] *= keep;
#pragma unroll
                for (int db = 0; db < DV / 16; ++db)
#pragma unroll
                    for (int i = 0; i < 4; ++i) oacc[db][qa][i] *= keep;
            }
        }
#pragma unroll
        for (int half = 0; half < 2; ++half) {
            u32x4_t ph[NQ], pl[NQ];
#pragma unroll
            for (int qa = 0; qa < NQ; ++qa) {
                const float ref = m[qa] == -INFINITY ? 0.f : m[qa];
#pragma unroll
                for (int kb2 = 0; kb2 < 2; ++kb2) {
                    float p[4];
#pragma unroll
                    for (int i = 0; i < 4; ++i) {
                        const float x = fmaf(sacc[2 * half + kb2][qa][i], to_exp2, -ref);
                        p[i] = seen(qa, 2 * half + kb2, i) ? __builtin_amdgcn_exp2f(x) : 0.f;
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

    fetch(0, 0);
    put(0);
    __syncthreads();
    for (int tile = 0; tile < ntiles; ++tile) {
        const int buf = kDirect ? tile & 1 : 0, next = kDirect ? buf ^ 1 : 0;
        if (tile + 1 < ntiles) fetch(tile + 1, next);                // (that buffer was read one tile ago, a barrier lies between)
        const int key0 = key_begin + tile * kBN;
        if (w_live && key0 <= w_last && key0 + kBN > w_lo) {
            if (key0 >= w_lo_all && key0 + kBN - 1 <= w_first) attend(std::false_type{}, key0, buf);
            else attend(std::true_type{}, key0, buf);
        }
        if (!kDirect) __syncthreads();
        if (tile + 1 < ntiles) put(next);
        __syncthreads();
    }
    if (!w_live) return;
#pragma unroll
    for (int qa = 0; qa < NQ; ++qa) {
        float l = lsum[qa];
        l += __shfl_xor(l, 16, 64);
        l += __shfl_xor(l, 32, 64);
        const int row = row0 + wave * 16 * NQ + 16 * qa + r;
        if (row >= lq) continue;
        const float inv = l > 0.f ? latent_gate<bf16_t>(a.gate, a.gate_stride, t0 + row, head) / (l + latent_sink(a.sinks, head, m[qa])) : 0.f;
        bf16_t *out = a.out + (static_cast<int64_t>(t0 + row) * a.heads + head) * a.vdim + 4 * g;
#pragma unroll
        for (int db = 0; db < DV / 16; ++db)
            if (16 * db + 4 * g < a.vdim) {
                const f32x4_t o = oacc[db][qa];
                *reinterpret_cast<u32x2_t *>(out + 16 * db) = u32x2_t{pack_bf16x2(o[0] * inv, o[1] * inv), pack_bf16x2(o[2] * inv, o[3] * inv)};
            }
    }
}

template <int DN, int DR, int DV, int NQ, bool kDirect>
static int launch_latent_prefill(const LatentPrefillArgs &a, int32_t n_seqs, int32_t max_q, hipStream_t s) {
    const int32_t q_tiles = (max_q + 64 * NQ - 1) / (64 * NQ);
    const int64_t wgs = static_cast<int64_t>(n_seqs) * q_tiles * a.heads;
    if (wgs > 0x7fffffffLL) return NVA_ERR_BAD_SHAPE;
    if (wgs == 0) return NVA_OK;
    hipLaunchKernelGGL((latent_prefill_kernel<DN, DR, DV, NQ, kDirect>), dim3(static_cast<uint32_t>(wgs)), dim3(256), 0, s, a, q_tiles);
    return launch_status();
}

}  // namespace nva

extern "C" int nva_latent_prepare(const void *x, int64_t x_row_stride, const void *q_norm_weight, const void *kv_norm_weight,
                                  const float *rope_cache, void *q_out, void *cache, const int32_t *slot_mapping, int64_t num_slots,
                                  const int32_t *cu_seqlens_q, const int32_t *seq_lens, const int32_t *token_seq, int32_t n_tokens,
                                  int32_t n_seqs, int32_t q_rank, int32_t kv_rank, int32_t rot_dim, int32_t max_position, float eps,
                                  int32_t dtype, void *stream) {
    using namespace nva;
    if (n_tokens < 0 || n_seqs < 0 || q_rank < 0 || max_position <= 0 || (cache && (kv_rank <= 0 || rot_dim < 0 || num_slots < 0))) return NVA_ERR_BAD_SHAPE;
    if (!known_dtype(dtype) || (cache && rot_dim % 2 != 0)) return NVA_ERR_UNSUPPORTED_GEOMETRY;
    if (n_tokens == 0) return NVA_OK;
    if (!x || (q_rank > 0 && (!q_norm_weight || !q_out)) || !seq_lens || (cache && (!kv_norm_weight || !slot_mapping || (rot_dim > 0 && !rope_cache)))) return NVA_ERR_NULL_POINTER;
    if (cu_seqlens_q && (!token_seq || n_seqs == 0)) return NVA_ERR_NULL_POINTER;
    if (!cu_seqlens_q && n_seqs != n_tokens) return NVA_ERR_BAD_SHAPE;
    if (x_row_stride < static_cast<int64_t>(q_rank) + (cache ? kv_rank + rot_dim : 0)) return NVA_ERR_BAD_STRIDE;
    LatentPrepareArgs a{};
    a.x = x; a.stride = x_row_stride; a.wq = q_norm_weight; a.wkv = kv_norm_weight; a.rope = rope_cache; a.q_out = q_out; a.cache = cache;
    a.slot_mapping = slot_mapping; a.num_slots = num_slots; a.rows = RowsOf{cu_seqlens_q, seq_lens, token_seq, n_tokens, n_seqs};
    a.q_rank = q_rank; a.rank = kv_rank; a.rot = rot_dim; a.max_position = max_position; a.eps = eps;
    const bool vector = q_rank % 8 == 0 && x_row_stride % 8 == 0 && aligned16(x) && aligned16(q_norm_weight) && aligned16(q_out) &&
                        (!cache || (kv_rank % 8 == 0 && rot_dim % 8 == 0 && aligned16(cache) && aligned16(kv_norm_weight)));
    const dim3 grid((n_tokens + 3) / 4), block(256);
    hipStream_t s = static_cast<hipStream_t>(stream);
    if (dtype == NVA_DTYPE_BF16) {
        if (vector) hipLaunchKernelGGL((latent_prepare_kernel<bf16_t, 8>), grid, block, 0, s, a);
        else hipLaunchKernelGGL((latent_prepare_kernel<bf16_t, 1>), grid, block, 0, s, a);
    } else {
        if (vector) hipLaunchKernelGGL((latent_prepare_kernel<float, 8>), grid, block, 0, s, a);
        else hipLaunchKernelGGL((latent_prepare_kernel<float, 1>), grid, block, 0, s, a);
    }
    return launch_status();
}

extern "C" size_t nva_latent_attn_workspace_bytes(int32_t n_tokens, int32_t num_heads, int32_t kv_rank, int32_t rot_dim,
                                                  int32_t max_blocks, int32_t block_size, int32_t window, int32_t dtype) {
    if (n_tokens <= 0 || num_heads <= 0 || kv_rank <= 0 || rot_dim < 0 || max_blocks < 0 || block_size <= 0 || window <= 0) return 0;
    if (!nva::latent_rows_ok(kv_rank, rot_dim, dtype)) return 0;
    const nva::LatentSplit sp = nva::plan_latent(n_tokens, num_heads, kv_rank, max_blocks, block_size, window);
    if (sp.splits == 1) return 0;
    return static_cast<size_t>(n_tokens) * sp.splits * num_heads * (kv_rank + 4) * sizeof(float);
}

extern "C" int nva_latent_attn(const void *q_latent, const void *q_rot, int64_t qr_row_stride, int64_t qr_head_stride, const void *gate,
                               int64_t gate_row_stride, const float *sinks, const float *rope_cache, const void *cache, const int32_t *block_tables,
                               int64_t bt_row_stride, int32_t max_blocks, const int32_t *cu_seqlens_q, const int32_t *seq_lens,
                               const int32_t *token_seq, void *out, void *workspace, size_t workspace_bytes, int32_t n_tokens,
                               int32_t n_seqs, int32_t num_heads, int32_t kv_rank, int32_t rot_dim, int32_t block_size,
                               int32_t num_blocks, int32_t window, int32_t max_position, float scale, int32_t dtype, void *stream) {
    using namespace nva;
    if (n_tokens < 0 || n_seqs < 0 || num_heads <= 0 || kv_rank <= 0 || rot_dim < 0 || num_blocks < 0 || max_blocks < 0 || window <= 0 || max_position <= 0)
        return NVA_ERR_BAD_SHAPE;
    const int shift = block_shift_of(block_size);
    if (shift < 0 || kv_rank + rot_dim > kLatentMax || rot_dim % 2 != 0 || !known_dtype(dtype)) return NVA_ERR_UNSUPPORTED_GEOMETRY;
    if (n_tokens == 0) return NVA_OK;
    if (!q_latent || !cache || !block_tables || !seq_lens || !out || (rot_dim > 0 && (!q_rot || !rope_cache))) return NVA_ERR_NULL_POINTER;
    if (cu_seqlens_q && (!token_seq || n_seqs == 0)) return NVA_ERR_NULL_POINTER;
    if (!cu_seqlens_q && n_seqs != n_tokens) return NVA_ERR_BAD_SHAPE;
    if (bt_row_stride < max_blocks || (gate && gate_row_stride < num_heads) || qr_head_stride < rot_dim || qr_row_stride < static_cast<int64_t>(num_heads - 1) * qr_head_stride + rot_dim)
        return NVA_ERR_BAD_STRIDE;
    if (static_cast<int64_t>(n_tokens) * num_heads / 4 > 0x7ffffff0LL) return NVA_ERR_BAD_SHAPE;
    LatentAttnArgs a{};
    a.q_lat = q_latent; a.q_rot = q_rot; a.qr_row = qr_row_stride; a.qr_head = qr_head_stride; a.gate = gate; a.gate_stride = gate_row_stride; a.sinks = sinks;
    a.rope = rope_cache; a.cache = cache; a.block_tables = block_tables; a.bt_stride = bt_row_stride; a.out = out;
    a.rows = RowsOf{cu_seqlens_q, seq_lens, token_seq, n_tokens, n_seqs}; a.heads = num_heads; a.rank = kv_rank; a.rot = rot_dim;
    a.block_shift = shift; a.num_blocks = num_blocks; a.max_blocks = max_blocks; a.window = window; a.max_position = max_position; a.scale = scale;
    hipStream_t s = static_cast<hipStream_t>(stream);
    if (latent_rows_ok(kv_rank, rot_dim, dtype) && qr_row_stride % 8 == 0 && qr_head_stride % 8 == 0 && aligned16(q_latent) && aligned16(q_rot) &&
        aligned16(cache) && aligned16(out)) {
        LatentSplit sp = plan_latent(n_tokens, num_heads, kv_rank, max_blocks, block_size, window);
        sp.partials = static_cast<float *>(workspace);
        if (sp.splits > 1) {
            if (!workspace) return NVA_ERR_NULL_POINTER;
            if (!aligned16(workspace)) return NVA_ERR_MISALIGNED;
            if (workspace_bytes < nva_latent_attn_workspace_bytes(n_tokens, num_heads, kv_rank, rot_dim, max_blocks, block_size, window, dtype))
                return NVA_ERR_WORKSPACE_TOO_SMALL;
        }
        const bool wide = num_heads > 16;
        if (kv_rank == 512 && rot_dim == 64) return launch_latent_rows<512, 64, 1, true>(a, sp, s);
        if (kv_rank <= 128) return wide ? launch_latent_rows<128, 64, 2, false>(a, sp, s) : launch_latent_rows<128, 64, 1, false>(a, sp, s);
        if (kv_rank <= 256) return wide ? launch_latent_rows<256, 64, 2, false>(a, sp, s) : launch_latent_rows<256, 64, 1, false>(a, sp, s);
        return launch_latent_rows<512, 64, 1, false>(a, sp, s);
    }
    const dim3 grid(static_cast<uint32_t>((static_cast<int64_t>(n_tokens) * num_heads + 3) / 4));
    if (dtype == NVA_DTYPE_BF16) hipLaunchKernelGGL((latent_attn_any_kernel<bf16_t>), grid, dim3(256), 0, s, a);
    else hipLaunchKernelGGL((latent_attn_any_kernel<float>), grid, dim3(256), 0, s, a);
    return launch_status();
}

extern "C" int nva_latent_gather(const void *cache, const int32_t *block_tables, int64_t bt_row_stride, int32_t max_blocks,
                                 const int32_t *key_cu, const int32_t *seq_lens, void *out, int32_t n_keys, int32_t n_seqs,
                                 int32_t row_width, int32_t block_size, int32_t num_blocks, int32_t dtype, void *stream) {
    using namespace nva;
    if (n_keys < 0 || n_seqs < 0 || row_width <= 0 || num_blocks < 0 || max_blocks < 0) return NVA_ERR_BAD_SHAPE;
    const int shift = block_shift_of(block_size);
    if (shift < 0 || !known_dtype(dtype)) return NVA_ERR_UNSUPPORTED_GEOMETRY;
    if (n_keys == 0) return NVA_OK;
    if (!cache || !block_tables || !key_cu || !seq_lens || !out) return NVA_ERR_NULL_POINTER;
    if (n_seqs == 0 || num_blocks == 0) return NVA_ERR_BAD_SHAPE;
    if (bt_row_stride < max_blocks) return NVA_ERR_BAD_STRIDE;
    const bool vector = row_width % 8 == 0 && aligned16(cache) && aligned16(out);
    const dim3 grid((n_keys + 3) / 4), block(256);
    hipStream_t s = static_cast<hipStream_t>(stream);
    if (dtype == NVA_DTYPE_BF16) {
        const bf16_t *c = static_cast<const bf16_t *>(cache);
        bf16_t *o = static_cast<bf16_t *>(out);
        if (vector) hipLaunchKernelGGL((latent_gather_kernel<bf16_t, 8>), grid, block, 0, s, c, block_tables, bt_row_stride, key_cu, seq_lens, o, n_keys, n_seqs, row_width, shift, num_blocks, max_blocks);
        else hipLaunchKernelGGL((latent_gather_kernel<bf16_t, 1>), grid, block, 0, s, c, block_tables, bt_row_stride, key_cu, seq_lens, o, n_keys, n_seqs, row_width, shift, num_blocks, max_blocks);
    } else {
        const float *c = static_cast<const float *>(cache);
        float *o = static_cast<float *>(out);
        if (vector) hipLaunchKernelGGL((latent_gather_kernel<float, 8>), grid, block, 0, s, c, block_tables, bt_row_stride, key_cu, seq_lens, o, n_keys, n_seqs, row_width, shift, num_blocks, max_blocks);
        else hipLaunchKernelGGL((latent_gather_kernel<float, 1>), grid, block, 0, s, c, block_tables, bt_row_stride, key_cu, seq_lens, o, n_keys, n_seqs, row_width, shift, num_blocks, max_blocks);
    }
    return launch_status();
}

extern "C" int nva_latent_prefill_supported(int32_t dim, int32_t rot_dim, int32_t v_dim, int32_t dtype) {
    return dtype == NVA_DTYPE_BF16 && dim > 0 && v_dim > 0 && rot_dim >= 0 && dim % 8 == 0 && rot_dim % 8 == 0 && v_dim % 8 == 0 && dim <= 256 &&
           rot_dim <= 128 && v_dim <= 256;
}

extern "C" int nva_latent_prefill(const void *q, int64_t q_row_stride, const void *kv, int64_t kv_row_stride, const void *k_rot,
                                  int64_t kr_row_stride, const void *gate, int64_t gate_row_stride, const float *sinks, const float *rope_cache,
                                  const int32_t *cu_seqlens_q, const int32_t *seq_lens, const int32_t *key_cu, void *out,
                                  int32_t n_tokens, int32_t n_seqs, int32_t max_seqlen_q, int32_t num_heads, int32_t dim, int32_t rot_dim,
                                  int32_t v_dim, int32_t window, int32_t max_position, float scale, int32_t dtype, void *stream) {
    using namespace nva;
    if (n_tokens < 0 || n_seqs < 0 || max_seqlen_q < 0 || num_heads <= 0 || dim <= 0 || rot_dim < 0 || v_dim <= 0 || window <= 0 || max_position <= 0) return NVA_ERR_BAD_SHAPE;
    if (!nva_latent_prefill_supported(dim, rot_dim, v_dim, dtype)) return NVA_ERR_UNSUPPORTED_GEOMETRY;
    if (n_tokens == 0 || n_seqs == 0) return NVA_OK;
    if (!q || !kv || !cu_seqlens_q || !seq_lens || !key_cu || !out || (rot_dim > 0 && (!k_rot || !rope_cache))) return NVA_ERR_NULL_POINTER;
    if (q_row_stride < static_cast<int64_t>(num_heads) * (dim + rot_dim) || kv_row_stride < static_cast<int64_t>(num_heads) * (dim + v_dim) ||
        kr_row_stride < rot_dim || (gate && gate_row_stride < num_heads) || q_row_stride % 8 != 0 || kv_row_stride % 8 != 0 || kr_row_stride % 8 != 0)
        return NVA_ERR_BAD_STRIDE;
    if (kv_row_stride > (1 << 24) || kr_row_stride > (1 << 24)) return NVA_ERR_BAD_STRIDE;      // offsets inside a tile are 32-bit
    if (!aligned16(q) || !aligned16(kv) || !aligned16(k_rot) || !aligned16(out)) return NVA_ERR_MISALIGNED;
    LatentPrefillArgs a{};
    a.q = static_cast<const bf16_t *>(q); a.q_stride = q_row_stride; a.kv = static_cast<const bf16_t *>(kv); a.kv_stride = kv_row_stride;
    a.k_rot = static_cast<const bf16_t *>(k_rot); a.kr_stride = kr_row_stride; a.gate = static_cast<const bf16_t *>(gate); a.gate_stride = gate_row_stride; a.sinks = sinks;
    a.rope = rope_cache; a.cu = cu_seqlens_q; a.klen = seq_lens; a.key_cu = key_cu; a.out = static_cast<bf16_t *>(out);
    a.heads = num_heads; a.dim = dim; a.rot = rot_dim; a.vdim = v_dim; a.window = window; a.max_position = max_position; a.scale = scale;
    hipStream_t s = static_cast<hipStream_t>(stream);
    if (dim == 128 && rot_dim == 64 && v_dim == 128) return launch_latent_prefill<128, 64, 128, 2, true>(a, n_seqs, max_seqlen_q, s);
    if (dim <= 64 && rot_dim <= 64 && v_dim <= 64) return launch_latent_prefill<64, 64, 64, 2, false>(a, n_seqs, max_seqlen_q, s);
    if (dim <= 128 && rot_dim <= 64 && v_dim <= 128) return launch_latent_prefill<128, 64, 128, 2, false>(a, n_seqs, max_seqlen_q, s);
    return launch_latent_prefill<256, 128, 256, 1, false>(a, n_seqs, max_seqlen_q, s);
}
