// Retention: linear attention with one fixed decay per head.
//   S_t = decay S_{t-1} + k_t v_t^T      o_t = S_t^T q_t
// q and k carry rotary positions, k is scaled by dim^-1/2; every head's o is divided by its root mean
// square and multiplied by silu of the gate projection.  The kernels take the projections as they
// come out of the matrix product (rows of q | k | v | gate) and do everything else.  State, rotated q
// and k, decays and norms are fp32; the state lives in slots [slot, head, dim, vdim].
#include "nva_elem.h"
#include "nva_matrix.h"

#include <math.h>

#include <algorithm>

namespace nva {

struct RetentionArgs {
    const void *x;                   // [n, 2 H dim + 2 H vdim]: q, k, v, gate
    int64_t stride;                  // elements
    float *state;                    // [num_slots, H, dim, vdim]
    const int32_t *slots;            // [n_seqs]
    const int32_t *cu;               // portions: [n_seqs + 1]; decode: null, row i is sequence i
    const int32_t *klen;             // tokens of every sequence, this step's included (decode: 0 = padded row)
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
        const int64_t pos = min(start + t, a.max_position - 1);
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

// Single tokens: one workgroup per (sequence, head) streams the state once -- read, decay, add k v^T, write,
// and the product with q on the way -- and finishes the head: norm, gate, store.  A thread owns four value
// columns (one 16-byte piece of a state row) of every kGroups-th row; eight rows are in flight at once.
// HBM: 2 * dim * vdim * 4 bytes per (sequence, head).
constexpr int kStepMaxDim = 512;

template <typename T>
__global__ __launch_bounds__(256) void retention_step_kernel(RetentionArgs a) {
    __shared__ float sh_q[kStepMaxDim], sh_k[kStepMaxDim];
    __shared__ __align__(16) float sh_red[1024];
    __shared__ float sh_w[4];
    const int seq = blockIdx.x / a.heads, head = blockIdx.x % a.heads;
    const int tid = threadIdx.x;
    const int start = a.klen[seq] - 1, slot = a.slots[seq];
    T *out = static_cast<T *>(a.out) + (static_cast<int64_t>(seq) * a.heads + head) * a.vdim;
    if (start < 0 || static_cast<uint32_t>(slot) >= static_cast<uint32_t>(a.num_slots)) {     // padded row
        for (int c = tid; c < a.vdim; c += 256) out[c] = Elem<T>::from_f32(0.f);
        return;
    }
    float *S = a.state + (static_cast<int64_t>(slot) * a.heads + head) * a.dim * a.vdim;
    const int per_row = a.vdim / 4, groups = 256 / per_row;
    const int piece = tid % per_row, group = tid / per_row;
    const bool mine = group < groups;
    // the first rows of the state are on their way while q and k are rotated
    constexpr int kAhead = 8;
    f32x4_t s[kAhead];
    auto fetch = [&](int r0) __attribute__((always_inline)) {
#pragma unroll
        for (int i = 0; i < kAhead; ++i) {
            const int r = r0 + i * groups;
            s[i] = f32x4_t{0.f, 0.f, 0.f, 0.f};
            if (mine && r < a.dim && start > 0)
                s[i] = __builtin_nontemporal_load(reinterpret_cast<const f32x4_t *>(S + static_cast<int64_t>(r) * a.vdim) + piece);
        }
    };
    fetch(group);
    const float decay = exp2f(a.log2_decay[head]);
    const int64_t qk = static_cast<int64_t>(a.heads) * a.dim;
    const T *row = static_cast<const T *>(a.x) + static_cast<int64_t>(seq) * a.stride;
    const T *q = row + static_cast<int64_t>(head) * a.dim, *k = q + qk;
    const T *v = row + 2 * qk + static_cast<int64_t>(head) * a.vdim, *gate = v + static_cast<int64_t>(a.heads) * a.vdim;
    const int64_t pos = min(start, a.max_position - 1);
    for (int i = tid; i < a.dim; i += 256) {
        float qv = Elem<T>::to_f32(q[i]), kv = Elem<T>::to_f32(k[i]);
        if (i < 2 * a.half) {
            const bool lower = i < a.half;
            const int f = lower ? i : i - a.half, other = lower ? i + a.half : i - a.half;
            const float c = a.rope[pos * (2 * a.half) + f], sn = a.rope[pos * (2 * a.half) + a.half + f];
            const float sg = lower ? -sn : sn;
            qv = qv * c + Elem<T>::to_f32(q[other]) * sg;
            kv = kv * c + Elem<T>::to_f32(k[other]) * sg;
        }
        sh_q[i] = qv;
        sh_k[i] = kv * a.k_scale;
    }
    f32x4_t vv = {0.f, 0.f, 0.f, 0.f};
    if (mine)
#pragma unroll
        for (int i = 0; i < 4; ++i) vv[i] = Elem<T>::to_f32(v[4 * piece + i]);
    __syncthreads();
    f32x4_t acc = {0.f, 0.f, 0.f, 0.f};
    for (int r0 = group; r0 < a.dim; r0 += kAhead * groups) {
#pragma unroll
        for (int i = 0; i < kAhead; ++i) {
            const int r = r0 + i * groups;
            if (mine && r < a.dim) {
                const float kr = sh_k[r], qr = sh_q[r];
#pragma unroll
                for (int j = 0; j < 4; ++j) {
                    s[i][j] = fmaf(decay, s[i][j], kr * vv[j]);
                    acc[j] = fmaf(s[i][j], qr, acc[j]);
                }
                __builtin_nontemporal_store(s[i], reinterpret_cast<f32x4_t *>(S + static_cast<int64_t>(r) * a.vdim) + piece);
            }
        }
        if (r0 + kAhead * groups < a.dim) fetch(r0 + kAhead * groups);
    }
    if (mine) *reinterpret_cast<f32x4_t *>(&sh_red[group * a.vdim + 4 * piece]) = acc;
    __syncthreads();
    float o[kStepMaxDim / 256], ss = 0.f;
#pragma unroll
    for (int i = 0; i < kStepMaxDim / 256; ++i) {
        const int c = tid + 256 * i;
        o[i] = 0.f;
        if (c < a.vdim)
            for (int g = 0; g < groups; ++g) o[i] += sh_red[g * a.vdim + c];
        ss = fmaf(o[i], o[i], ss);
    }
    ss = wave_sum(ss);
    if ((tid & 63) == 0) sh_w[tid >> 6] = ss;
    __syncthreads();
    const float inv = rsqrtf(((sh_w[0] + sh_w[1]) + (sh_w[2] + sh_w[3])) / static_cast<float>(a.vdim) + a.eps);
#pragma unroll
    for (int i = 0; i < kStepMaxDim / 256; ++i) {
        const int c = tid + 256 * i;
        if (c < a.vdim) {
            const float z = Elem<T>::to_f32(gate[c]);
            out[c] = Elem<T>::from_f32(o[i] * inv * (z * sigmoid_of<T>(z)));
        }
    }
}

// ---- portions, bf16, on the matrix cores -----------------------------------------------------------
// A workgroup walks one (sequence, head) -- or one segment of it -- in chunks of 32 tokens.  With S the
// state before a chunk and i, j places in it,
//     o_i = decay^{i+1} S^T q_i + sum_{j <= i} decay^{i-j} (q_i . k_j) v_j
//     S'  = decay^L S + sum_j decay^{L-1-j} k_j v_j^T                      (L tokens in the chunk)
// which is four small matrix products.  Wavefront w keeps its 16 NV value columns of S in accumulator
// registers for the whole walk; as accumulators hold S with the value column in the lane, they are also
// the first operand of S^T q (register i of lane l: row 4 (l / 16) + i of a 16-row block, two blocks make
// the 32 inner indices; q is read in that order).
// Everything that is fp32 here -- rotated q and k, decayed scores, the state, decayed v -- enters a product
// as the sum of two bf16 numbers (high x high, high x low, low x high: 16 bits of mantissa); v is
// bf16 to begin with.  Accumulation is fp32.
// Long sequences are cut into segments so that the machine fills: the segments' own sums (kSums) are formed
// first, a scan over the segments turns them into the state each one starts from, then all run at once.
constexpr int kRetChunk = 32;
// token of a chunk that inner index 4 s + a of 16-lane group g stands for.  Groups 0 and 1, whose LDS
// reads go together, take every other token: with rows 16 bytes off a multiple of 256 these lie in
// different banks.
__device__ __forceinline__ int chunk_token(int g, int s, int a) { return 2 * (4 * (g & 1) + a) + (g >> 1) + 16 * s; }

struct SegmentArgs {
    float *sums;         // [n_seqs, segments, H, dim, vdim] (segments > 1)
    int32_t segments, length;
};

template <int DK, int NV, bool kSums>
__global__ __launch_bounds__(256, DK * NV > 256 ? 1 : 2) void retention_chunk_kernel(const RetentionArgs a, const SegmentArgs sg) {
    constexpr int kC = kRetChunk, kDB = DK / 16, kPitch = DK * 2 + 16, kVW = 64 * NV, kVPitch = kVW * 2 + 16, kPPitch = kC * 2 + 16;
    constexpr int kQ = 0, kK = kSums ? 0 : 2 * kC * kPitch, kV = kK + 2 * kC * kPitch, kP = kV + kC * kVPitch;
    __shared__ __attribute__((aligned(16))) unsigned char smem[kP + (kSums ? 0 : 2 * kC * kPPitch)];
    __shared__ float sh_ss[4][kC];
    const lds_char_ptr lds = (lds_char_ptr)(&smem[0]);
    const int tid = threadIdx.x, lane = tid & 63;
    const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
    const int r = lane & 15, g = lane >> 4;
    const int head = blockIdx.x % a.heads;
    const int seg = blockIdx.x / a.heads % sg.segments, seq = blockIdx.x / a.heads / sg.segments;
    const int first = a.cu[seq], count = a.cu[seq + 1] - first, start = a.klen[seq] - count;
    const int t_begin = seg * sg.length, t_end = min(count, t_begin + sg.length);
    if (t_begin >= count || start < 0) return;
    if (kSums && t_end == count) return;                 // nothing follows the last segment
    const int slot = a.slots[seq];
    const bool have_slot = static_cast<uint32_t>(slot) < static_cast<uint32_t>(a.num_slots);
    const int64_t state_size = static_cast<int64_t>(a.dim) * a.vdim;
    float *slot_state = a.state + (static_cast<int64_t>(have_slot ? slot : 0) * a.heads + head) * state_size;
    float *seg_state = sg.sums + ((static_cast<int64_t>(seq) * sg.segments + seg) * a.heads + head) * state_size;
    const float l2 = a.log2_decay[head];
    const int v0 = wave * 16 * NV;                       // this wavefront's first value column

    f32x4_t S[kDB][NV];
    {
        const float *src = sg.segments > 1 ? seg_state : slot_state;
        const bool load = !kSums && (sg.segments > 1 || (have_slot && start > 0));
#pragma unroll
        for (int db = 0; db < kDB; ++db)
#pragma unroll
            for (int vb = 0; vb < NV; ++vb)
#pragma unroll
                for (int i = 0; i < 4; ++i) {
                    const int d = 16 * db + 4 * g + i, v = v0 + 16 * vb + r;
                    S[db][vb][i] = load && d < a.dim && v < a.vdim ? src[static_cast<int64_t>(d) * a.vdim + v] : 0.f;
                }
    }
    // decay factors that do not change from chunk to chunk
    const int s_qb = wave >> 1, s_kb = wave & 1;         // the block of scores this wavefront computes
    float dmat[4], gq[2], vfac[8];
#pragma unroll
    for (int i = 0; i < 4; ++i) {
        const int lag = 16 * s_qb + r - (16 * s_kb + 4 * g + i);
        dmat[i] = lag >= 0 ? __builtin_amdgcn_exp2f(l2 * lag) : 0.f;
    }
#pragma unroll
    for (int qb = 0; qb < 2; ++qb) gq[qb] = __builtin_amdgcn_exp2f(l2 * (16 * qb + r + 1));
#pragma unroll
    for (int e = 0; e < 8; ++e) vfac[e] = __builtin_amdgcn_exp2f(l2 * (kC - 1 - chunk_token(g, e >> 2, e & 3)));
    const float inv_vdim = 1.0f / static_cast<float>(a.vdim);
    float g_chunk = __builtin_amdgcn_exp2f(l2 * kC);

    const int64_t qk = static_cast<int64_t>(a.heads) * a.dim;
    const bf16_t *xq = static_cast<const bf16_t *>(a.x) + static_cast<int64_t>(head) * a.dim;
    const bf16_t *xv = static_cast<const bf16_t *>(a.x) + 2 * qk + static_cast<int64_t>(head) * a.vdim;
    const bf16_t *xg = xv + static_cast<int64_t>(a.heads) * a.vdim;
    const int pairs = a.half / 8, units = DK / 8 - pairs;            // per row: pairs of pieces that rotate, then single pieces
    struct Unit { int e0, e1; bool pair; };
    auto unit_of = [&](int w) __attribute__((always_inline)) -> Unit {
        const bool pair = w < pairs;
        const int e0 = pair ? 8 * w : 2 * a.half + 8 * (w - pairs);
        return Unit{e0, pair ? e0 + a.half : e0, pair};
    };
    // a thread's first unit of q and k and its pieces of v (32 rows of 64 NV columns) are loaded one chunk ahead
    u32x4_t rq0, rq1, rk0, rk1, rv[NV];
    const int my_row = tid / units;
    const Unit my_unit = unit_of(tid % units);
    auto fetch = [&](int row, const Unit &w, int t0) __attribute__((always_inline)) {
        rq0 = rq1 = rk0 = rk1 = u32x4_t{0, 0, 0, 0};
        if (row < kC && t0 + row < t_end && w.e0 < a.dim) {
            const bf16_t *x = xq + static_cast<int64_t>(first + t0 + row) * a.stride;
            if (!kSums) {
                rq0 = *reinterpret_cast<const u32x4_t *>(x + w.e0);
                rq1 = *reinterpret_cast<const u32x4_t *>(x + w.e1);
            }
            rk0 = *reinterpret_cast<const u32x4_t *>(x + qk + w.e0);
            rk1 = *reinterpret_cast<const u32x4_t *>(x + qk + w.e1);
        }
    };
    float rcos[8], rsin[8];
    auto fetch_turn = [&](int row, const Unit &w, int t0) __attribute__((always_inline)) {
        if (w.pair) {
            const float *cs = a.rope + static_cast<int64_t>(min(start + t0 + row, a.max_position - 1)) * (2 * a.half) + w.e0;
            load_f32<float, 8>(cs, rcos);
            load_f32<float, 8>(cs + a.half, rsin);
        }
    };
    auto fetch_v = [&](int t0) __attribute__((always_inline)) {
#pragma unroll
        for (int i = 0; i < NV; ++i) {
            const int p = i * 256 + tid, row = p / (kVW / 8), e = p % (kVW / 8) * 8;
            rv[i] = u32x4_t{0, 0, 0, 0};
            if (t0 + row < t_end && e < a.vdim) rv[i] = *reinterpret_cast<const u32x4_t *>(xv + static_cast<int64_t>(first + t0 + row) * a.stride + e);
        }
    };
    fetch(my_row, my_unit, t_begin);
    fetch_turn(my_row, my_unit, t_begin);
    fetch_v(t_begin);

    for (int t0 = t_begin; t0 < t_end; t0 += kC) {
        const int L = min(kC, t_end - t0);
        // ---- q and k: rotate, split; v; all into LDS ------------------------------------------------
        auto place = [&](const u32x4_t &p0, const u32x4_t &p1, bool pair, const float (&c)[8], const float (&s)[8], float scale,
                         lds_char_ptr dst0, lds_char_ptr dst1) __attribute__((always_inline)) {
            float x0[8], x1[8], y[8];
            u32x4_t hi, lo;
            unpack8(make_uint4(p0[0], p0[1], p0[2], p0[3]), x0);
            if (pair) {
                unpack8(make_uint4(p1[0], p1[1], p1[2], p1[3]), x1);
#pragma unroll
                for (int i = 0; i < 8; ++i) y[i] = x1[i] * c[i] + x0[i] * s[i];
                split8(y, hi, lo);
                *(lds_u32x4_ptr)dst1 = hi;
                *(lds_u32x4_ptr)(dst1 + kC * kPitch) = lo;
#pragma unroll
                for (int i = 0; i < 8; ++i) y[i] = x0[i] * c[i] - x1[i] * s[i];
            } else {
#pragma unroll
                for (int i = 0; i < 8; ++i) y[i] = x0[i] * scale;
            }
            split8(y, hi, lo);
            *(lds_u32x4_ptr)dst0 = hi;
            *(lds_u32x4_ptr)(dst0 + kC * kPitch) = lo;
        };
        auto place_unit = [&](int row, const Unit &w) __attribute__((always_inline)) {
            float c[8], s[8];
#pragma unroll
            for (int i = 0; i < 8; ++i) { c[i] = rcos[i]; s[i] = rsin[i]; }
            const lds_char_ptr d0 = lds + row * kPitch + 2 * w.e0, d1 = lds + row * kPitch + 2 * w.e1;
            if (!kSums) place(rq0, rq1, w.pair, c, s, 1.0f, d0 + kQ, d1 + kQ);
            if (w.pair)
#pragma unroll
                for (int i = 0; i < 8; ++i) { c[i] *= a.k_scale; s[i] *= a.k_scale; }
            place(rk0, rk1, w.pair, c, s, a.k_scale, d0 + kK, d1 + kK);
        };
        if (tid < kC * units) place_unit(my_row, my_unit);
        for (int u = tid + 256; u < kC * units; u += 256) {          // (sizes with more than one unit per thread)
            const int row = u / units;
            const Unit w = unit_of(u % units);
            fetch(row, w, t0);
            fetch_turn(row, w, t0);
            place_unit(row, w);
        }
#pragma unroll
        for (int i = 0; i < NV; ++i) {
            const int p = i * 256 + tid;
            *(lds_u32x4_ptr)(lds + kV + p / (kVW / 8) * kVPitch + p % (kVW / 8) * 16) = rv[i];
        }
        __syncthreads();
        if (t0 + kC < t_end) {
            fetch(my_row, my_unit, t0 + kC);
            fetch_v(t0 + kC);
        }
        if (L < kC) {                                    // the last chunk of the segment
#pragma unroll
            for (int e = 0; e < 8; ++e) {
                const int back = L - 1 - chunk_token(g, e >> 2, e & 3);
                vfac[e] = back >= 0 ? __builtin_amdgcn_exp2f(l2 * back) : 0.f;
            }
            g_chunk = __builtin_amdgcn_exp2f(l2 * L);
        }
        f32x4_t O[NV][2];
        if (!kSums) {
            // operands in the accumulators' inner order: 32 ks + 4 g + [0, 4) and 16 further on
            auto row_frag = [&](int at, int row, int ks) __attribute__((always_inline)) -> u32x4_t {
                typedef __attribute__((address_space(3))) u32x2_t *lds_u32x2_ptr;
                const lds_char_ptr p = lds + at + row * kPitch + 64 * ks + 8 * g;
                const u32x2_t x = *(lds_u32x2_ptr)p, y = *(lds_u32x2_ptr)(p + 32);
                return u32x4_t{x[0], x[1], y[0], y[1]};
            };
#pragma unroll
            for (int vb = 0; vb < NV; ++vb) O[vb][0] = O[vb][1] = f32x4_t{0.f, 0.f, 0.f, 0.f};
            f32x4_t sc = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
            for (int ks = 0; ks < DK / 32; ++ks) {
                u32x4_t qh[2], ql[2];
#pragma unroll
                for (int qb = 0; qb < 2; ++qb) {
                    qh[qb] = row_frag(kQ, 16 * qb + r, ks);
                    ql[qb] = row_frag(kQ + kC * kPitch, 16 * qb + r, ks);
                }
                if (s_qb >= s_kb) {                      // (wave-uniform)
                    const u32x4_t kh = row_frag(kK, 16 * s_kb + r, ks), kl = row_frag(kK + kC * kPitch, 16 * s_kb + r, ks);
                    const u32x4_t sh = s_qb ? qh[1] : qh[0], sl = s_qb ? ql[1] : ql[0];
                    sc = mfma16(kh, sh, sc);
                    sc = mfma16(kh, sl, sc);
                    sc = mfma16(kl, sh, sc);
                }
#pragma unroll
                for (int vb = 0; vb < NV; ++vb) {
                    u32x4_t hi, lo;
                    const float f[8] = {S[2 * ks][vb][0], S[2 * ks][vb][1], S[2 * ks][vb][2], S[2 * ks][vb][3],
                                        S[2 * ks + 1][vb][0], S[2 * ks + 1][vb][1], S[2 * ks + 1][vb][2], S[2 * ks + 1][vb][3]};
                    split8(f, hi, lo);
#pragma unroll
                    for (int qb = 0; qb < 2; ++qb) {
                        O[vb][qb] = mfma16(hi, qh[qb], O[vb][qb]);
                        O[vb][qb] = mfma16(hi, ql[qb], O[vb][qb]);
                        O[vb][qb] = mfma16(lo, qh[qb], O[vb][qb]);
                    }
                }
            }
#pragma unroll
            for (int vb = 0; vb < NV; ++vb)
#pragma unroll
                for (int qb = 0; qb < 2; ++qb)
#pragma unroll
                    for (int i = 0; i < 4; ++i) O[vb][qb][i] *= gq[qb];
            // decayed scores to LDS: row = query, columns in chunk_token order.  Keys 4 g .. 4 g + 3 of block
            // s_kb: the even two are neighbours there, and so are the odd two, 16 columns on
            uint32_t he, le, ho, lo;
            split_pair(sc[0] * dmat[0], sc[2] * dmat[2], he, le);
            split_pair(sc[1] * dmat[1], sc[3] * dmat[3], ho, lo);
            typedef __attribute__((address_space(3))) uint32_t *lds_u32_ptr;
            const lds_char_ptr p = lds + kP + (16 * s_qb + r) * kPPitch + 2 * (8 * (g >> 1) + 4 * s_kb + 2 * (g & 1));
            *(lds_u32_ptr)p = he;
            *(lds_u32_ptr)(p + 32) = ho;
            *(lds_u32_ptr)(p + kC * kPPitch) = le;
            *(lds_u32_ptr)(p + kC * kPPitch + 32) = lo;
            __syncthreads();
        }
        // ---- v^T fragments: the second product's first operand and, decayed, the state's second ------
        auto token_frag = [&](int at, int pitch, int col) __attribute__((always_inline)) -> u32x4_t {
            const lds_char_ptr p = lds + at + chunk_token(g, 0, r >> 2) * pitch + 2 * (col + 4 * (r & 3));
            const s16x4_t x = __builtin_amdgcn_ds_read_tr16_b64_v4i16((lds_s16x4_ptr)p);
            const s16x4_t y = __builtin_amdgcn_ds_read_tr16_b64_v4i16((lds_s16x4_ptr)(p + 16 * pitch));
            return __builtin_bit_cast(u32x4_t, __builtin_shufflevector(x, y, 0, 1, 2, 3, 4, 5, 6, 7));
        };
        u32x4_t vf[NV];
#pragma unroll
        for (int vb = 0; vb < NV; ++vb) vf[vb] = token_frag(kV, kVPitch, v0 + 16 * vb);
        if (!kSums) {
#pragma unroll
            for (int qb = 0; qb < 2; ++qb) {
                const lds_char_ptr p = lds + kP + (16 * qb + r) * kPPitch + 16 * g;
                const u32x4_t ph = *(lds_u32x4_ptr)p, pl = *(lds_u32x4_ptr)(p + kC * kPPitch);
#pragma unroll
                for (int vb = 0; vb < NV; ++vb) {
                    O[vb][qb] = mfma16(vf[vb], ph, O[vb][qb]);
                    O[vb][qb] = mfma16(vf[vb], pl, O[vb][qb]);
                }
            }
        }
        u32x4_t vh[NV], vl[NV];
#pragma unroll
        for (int vb = 0; vb < NV; ++vb) {
            float f[8];
            unpack8(make_uint4(vf[vb][0], vf[vb][1], vf[vb][2], vf[vb][3]), f);
#pragma unroll
            for (int e = 0; e < 8; ++e) f[e] *= vfac[e];
            split8(f, vh[vb], vl[vb]);
        }
        // what the end of this chunk and the start of the next one wait for: gates, angles
        u32x2_t gate[kSums ? 1 : 2][NV];
        if (!kSums) {
#pragma unroll
            for (int qb = 0; qb < 2; ++qb)
#pragma unroll
                for (int vb = 0; vb < NV; ++vb) {
                    const int v = v0 + 16 * vb + 4 * g;
                    if (16 * qb + r < L && v < a.vdim)
                        gate[qb][vb] = *reinterpret_cast<const u32x2_t *>(xg + static_cast<int64_t>(first + t0 + 16 * qb + r) * a.stride + v);
                }
        }
        if (t0 + kC < t_end) fetch_turn(my_row, my_unit, t0 + kC);
#pragma unroll
        for (int db = 0; db < kDB; ++db) {
            const u32x4_t kh = token_frag(kK, kPitch, 16 * db), kl = token_frag(kK + kC * kPitch, kPitch, 16 * db);
#pragma unroll
            for (int vb = 0; vb < NV; ++vb) {
#pragma unroll
                for (int i = 0; i < 4; ++i) S[db][vb][i] *= g_chunk;
                S[db][vb] = mfma16(kh, vh[vb], S[db][vb]);
                S[db][vb] = mfma16(kh, vl[vb], S[db][vb]);
                S[db][vb] = mfma16(kl, vh[vb], S[db][vb]);
            }
        }
        if (!kSums) {
            // ---- head norm (value columns are spread over registers, lane groups and wavefronts), gate, store
#pragma unroll
            for (int qb = 0; qb < 2; ++qb) {
                float ss = 0.f;
#pragma unroll
                for (int vb = 0; vb < NV; ++vb)
#pragma unroll
                    for (int i = 0; i < 4; ++i) ss = fmaf(O[vb][qb][i], O[vb][qb][i], ss);
                ss += __shfl_xor(ss, 16, 64);
                ss += __shfl_xor(ss, 32, 64);
                if (g == 0) sh_ss[wave][16 * qb + r] = ss;
            }
        }
        __syncthreads();
        if (!kSums) {
#pragma unroll
            for (int qb = 0; qb < 2; ++qb) {
                const int row = 16 * qb + r;
                const float ss = (sh_ss[0][row] + sh_ss[1][row]) + (sh_ss[2][row] + sh_ss[3][row]);
                const float inv = rsqrtf(fmaf(ss, inv_vdim, a.eps));
                if (row >= L) continue;
                const int64_t t = first + t0 + row;
                bf16_t *out = static_cast<bf16_t *>(a.out) + (t * a.heads + head) * a.vdim;
#pragma unroll
                for (int vb = 0; vb < NV; ++vb) {
                    const int v = v0 + 16 * vb + 4 * g;
                    if (v < a.vdim) {
                        const u32x2_t z = gate[qb][vb];
                        const float zf[4] = {bf16lo_to_f32(z[0]), bf16hi_to_f32(z[0]), bf16lo_to_f32(z[1]), bf16hi_to_f32(z[1])};
                        float y[4];
#pragma unroll
                        for (int i = 0; i < 4; ++i) y[i] = O[vb][qb][i] * inv * (zf[i] * sigmoid_of<bf16_t>(zf[i]));
                        *reinterpret_cast<u32x2_t *>(out + v) = u32x2_t{pack_bf16x2(y[0], y[1]), pack_bf16x2(y[2], y[3])};
                    }
                }
            }
        }
    }
    if (!kSums && (t_end < count || !have_slot)) return;
    float *dst = kSums ? seg_state : slot_state;
#pragma unroll
    for (int db = 0; db < kDB; ++db)
#pragma unroll
        for (int vb = 0; vb < NV; ++vb)
#pragma unroll
            for (int i = 0; i < 4; ++i) {
                const int d = 16 * db + 4 * g + i, v = v0 + 16 * vb + r;
                if (d < a.dim && v < a.vdim) dst[static_cast<int64_t>(d) * a.vdim + v] = S[db][vb][i];
            }
}

// Replaces every segment's own sums by the state the segment starts from; one thread per four state elements
// (the value size is a multiple of 8).
__global__ __launch_bounds__(256) void retention_segment_scan_kernel(const RetentionArgs a, const SegmentArgs sg) {
    const int head = blockIdx.x % a.heads, seq = blockIdx.x / a.heads;
    const int64_t size = static_cast<int64_t>(a.dim) * a.vdim;
    const int64_t e = (static_cast<int64_t>(blockIdx.y) * 256 + threadIdx.x) * 4;
    const int count = a.cu[seq + 1] - a.cu[seq], start = a.klen[seq] - count;
    if (e >= size || count <= 0 || start < 0) return;
    const int slot = a.slots[seq];
    const bool carried = start > 0 && static_cast<uint32_t>(slot) < static_cast<uint32_t>(a.num_slots);
    f32x4_t run = {0.f, 0.f, 0.f, 0.f};
    if (carried) run = *reinterpret_cast<const f32x4_t *>(a.state + (static_cast<int64_t>(slot) * a.heads + head) * size + e);
    const float decay = exp2f(a.log2_decay[head] * static_cast<float>(sg.length));
    const int segments = min(sg.segments, (count - 1) / sg.length + 1);
    float *p = sg.sums + (static_cast<int64_t>(seq) * sg.segments * a.heads + head) * size + e;
    const int64_t step = static_cast<int64_t>(a.heads) * size;
    constexpr int kAhead = 16;                            // loads in flight together
    for (int s0 = 0; s0 < segments; s0 += kAhead) {
        f32x4_t own[kAhead];
#pragma unroll
        for (int i = 0; i < kAhead; ++i) {
            own[i] = f32x4_t{0.f, 0.f, 0.f, 0.f};
            if (s0 + i + 1 < segments) own[i] = *reinterpret_cast<const f32x4_t *>(p + (s0 + i) * step);
        }
#pragma unroll
        for (int i = 0; i < kAhead; ++i)
            if (s0 + i < segments) {
                *reinterpret_cast<f32x4_t *>(p + (s0 + i) * step) = run;
#pragma unroll
                for (int j = 0; j < 4; ++j) run[j] = fmaf(decay, run[j], own[i][j]);
            }
    }
}

// Segments of a call: enough (sequence, head, segment) workgroups for the machine, none shorter than 256
// tokens.  Depends on shapes only.
static SegmentArgs plan_segments(int32_t n_seqs, int32_t heads, int32_t max_q) {
    SegmentArgs sg{};
    const int64_t walks = std::max<int64_t>(1, static_cast<int64_t>(n_seqs) * heads);
    const int64_t want = std::min<int64_t>(std::max<int64_t>(1, 512 / walks), std::max(1, max_q / 256));
    const int64_t length = (max_q + want - 1) / want;
    sg.length = static_cast<int32_t>(std::max<int64_t>(kRetChunk, (length + kRetChunk - 1) / kRetChunk * kRetChunk));
    sg.segments = std::max(1, (max_q + sg.length - 1) / sg.length);
    return sg;
}

template <int DK, int NV>
static int launch_chunks(const RetentionArgs &a, const SegmentArgs &sg, hipStream_t s) {
    const dim3 grid(static_cast<uint32_t>(a.n_seqs) * sg.segments * a.heads), block(256);
    if (sg.segments > 1) {
        hipLaunchKernelGGL((retention_chunk_kernel<DK, NV, true>), grid, block, 0, s, a, sg);
        int rc = launch_status();
        if (rc != NVA_OK) return rc;
        hipLaunchKernelGGL(retention_segment_scan_kernel, dim3(a.n_seqs * a.heads, (a.dim * a.vdim + 1023) / 1024), block, 0, s, a, sg);
        rc = launch_status();
        if (rc != NVA_OK) return rc;
    }
    hipLaunchKernelGGL((retention_chunk_kernel<DK, NV, false>), grid, block, 0, s, a, sg);
    return launch_status();
}

// Sizes the chunked form is built for: everything vectors can hold with the state in registers.
static bool chunks_ok(int32_t dim, int32_t vdim, int32_t half) {
    return dim % 8 == 0 && vdim % 8 == 0 && half % 8 == 0 && ((dim <= 128 && vdim <= 256) || (dim <= 256 && vdim <= 128));
}

template <int DK>
static int launch_chunks_dk(const RetentionArgs &a, const SegmentArgs &sg, hipStream_t s) {
    if (a.vdim <= 64) return launch_chunks<DK, 1>(a, sg, s);
    if (a.vdim <= 128) return launch_chunks<DK, 2>(a, sg, s);
    if constexpr (DK <= 128) return launch_chunks<DK, 4>(a, sg, s);
    return NVA_ERR_UNSUPPORTED_GEOMETRY;
}

template <typename T>
static int launch_scan_any(const RetentionArgs &a, hipStream_t s) {
    hipLaunchKernelGGL((retention_scan_any_kernel<T>), dim3(a.n_seqs * a.heads), dim3(256), 0, s, a);
    return launch_status();
}

}  // namespace nva

extern "C" size_t nva_retention_workspace_bytes(int32_t n_seqs, int32_t max_seqlen_q, int32_t num_heads, int32_t qk_dim,
                                                int32_t v_dim, int32_t rot_dims, int32_t dtype) {
    if (n_seqs <= 0 || max_seqlen_q <= 0 || num_heads <= 0 || qk_dim <= 0 || v_dim <= 0 || rot_dims < 0) return 0;
    if (dtype != NVA_DTYPE_BF16 || !nva::chunks_ok(qk_dim, v_dim, rot_dims / 2)) return 0;
    const nva::SegmentArgs sg = nva::plan_segments(n_seqs, num_heads, max_seqlen_q);
    if (sg.segments == 1) return 0;
    return static_cast<size_t>(n_seqs) * sg.segments * num_heads * qk_dim * v_dim * sizeof(float);
}

extern "C" int nva_retention(const void *qkvg, int64_t row_stride, float *state, const int32_t *state_slots_of_seq,
                             const int32_t *cu_seqlens_q, const int32_t *seq_lens,
                             const float *rope_cache, const float *log2_decay, void *out, void *workspace,
                             size_t workspace_bytes, int32_t n_tokens, int32_t n_seqs,
                             int32_t max_seqlen_q, int32_t num_heads, int32_t qk_dim, int32_t v_dim, int32_t rot_dims,
                             int32_t max_position, int32_t num_state_slots, float k_scale, float eps, int32_t dtype,
                             void *stream) {
    using namespace nva;
    if (n_tokens < 0 || n_seqs < 0 || max_seqlen_q < 0 || num_heads <= 0 || qk_dim <= 0 || v_dim <= 0 || rot_dims < 0 ||
        rot_dims > qk_dim || max_position <= 0 || num_state_slots < 0)
        return NVA_ERR_BAD_SHAPE;
    if (rot_dims % 2 != 0 || qk_dim > kScanMaxDim || v_dim > kScanMaxDim || !known_dtype(dtype)) return NVA_ERR_UNSUPPORTED_GEOMETRY;
    if (n_tokens == 0 || n_seqs == 0) return NVA_OK;
    if (!qkvg || !state || !state_slots_of_seq || !seq_lens || !log2_decay || !out) return NVA_ERR_NULL_POINTER;
    if (rot_dims > 0 && !rope_cache) return NVA_ERR_NULL_POINTER;
    if (cu_seqlens_q == nullptr && n_seqs != n_tokens) return NVA_ERR_BAD_SHAPE;
    if (row_stride < 2 * static_cast<int64_t>(num_heads) * (qk_dim + v_dim)) return NVA_ERR_BAD_STRIDE;
    if (static_cast<int64_t>(n_seqs) * num_heads > 0x7fffffffLL) return NVA_ERR_BAD_SHAPE;
    RetentionArgs a{};
    a.x = qkvg; a.stride = row_stride; a.state = state; a.slots = state_slots_of_seq; a.cu = cu_seqlens_q; a.klen = seq_lens;
    a.rope = rope_cache; a.log2_decay = log2_decay; a.out = out; a.n = n_tokens; a.n_seqs = n_seqs;
    a.heads = num_heads; a.dim = qk_dim; a.vdim = v_dim; a.half = rot_dims / 2; a.num_slots = num_state_slots;
    a.max_position = max_position; a.k_scale = k_scale; a.eps = eps;
    hipStream_t s = static_cast<hipStream_t>(stream);
    if (cu_seqlens_q == nullptr && v_dim % 4 == 0 && aligned16(state)) {
        const dim3 grid(static_cast<uint32_t>(n_seqs) * num_heads), block(256);
        if (dtype == NVA_DTYPE_BF16) hipLaunchKernelGGL((retention_step_kernel<bf16_t>), grid, block, 0, s, a);
        else hipLaunchKernelGGL((retention_step_kernel<float>), grid, block, 0, s, a);
        return launch_status();
    }
    if (cu_seqlens_q != nullptr && dtype == NVA_DTYPE_BF16 && chunks_ok(qk_dim, v_dim, a.half) && row_stride % 8 == 0 &&
        aligned16(state) && aligned16(qkvg) && aligned16(out) && aligned16(rope_cache)) {
        SegmentArgs sg = plan_segments(n_seqs, num_heads, max_seqlen_q);
        sg.sums = static_cast<float *>(workspace);
        if (sg.segments > 1) {
            if (!workspace) return NVA_ERR_NULL_POINTER;
            if (!aligned16(workspace)) return NVA_ERR_MISALIGNED;
            if (workspace_bytes < nva_retention_workspace_bytes(n_seqs, max_seqlen_q, num_heads, qk_dim, v_dim, rot_dims, dtype))
                return NVA_ERR_WORKSPACE_TOO_SMALL;
        }
        if (static_cast<int64_t>(n_seqs) * sg.segments * num_heads > 0x7fffffffLL) return NVA_ERR_BAD_SHAPE;
        if (qk_dim <= 64) return launch_chunks_dk<64>(a, sg, s);
        if (qk_dim <= 128) return launch_chunks_dk<128>(a, sg, s);
        return launch_chunks_dk<256>(a, sg, s);
    }
    return dtype == NVA_DTYPE_BF16 ? launch_scan_any<bf16_t>(a, s) : launch_scan_any<float>(a, s);
}
