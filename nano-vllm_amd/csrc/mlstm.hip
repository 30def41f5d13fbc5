// Matrix memory with exponential gates (the mLSTM of xLSTM).  Per head, with log gates i_t and f_t <= 0:
//   m_t = max(f_t + m_{t-1}, i_t)                                     (m_0 = 0)
//   S_t = e^{f_t + m_{t-1} - m_t} S_{t-1} + e^{i_t - m_t} k_t v_t^T     n_t likewise with k_t alone
//   o_t = S_t^T q_t / (max(|n_t . q_t|, e^{-m_t}) + guard)
//   i = cap tanh((z_i + b_i) / cap)      f = log sigmoid(cap tanh((z_f + b_f) / cap))
// Every head's o is divided by its root mean square, multiplied by a weight and by the sigmoid of a gate
// projection.  The kernels take the projections as they come out of the matrix products (rows of
// q | k | v | gate, and z in fp32) and do everything else.  S, n and m are fp32 and live in slots.
#include "nva_elem.h"
#include "nva_matrix.h"

#include <math.h>

#include <algorithm>

namespace nva {

struct MlstmArgs {
    const void *x;                   // [n, 2 H dim + 2 H vdim]: q, k, v, gate
    int64_t stride;                  // elements
    const float *z;                  // [n, 2 H] dense: input gates, forget gates
    const float *bias;               // [2 H]
    const void *weight;              // [H vdim], of the head norm
    float *state, *mass, *top;       // [num_slots, H, dim, vdim], [num_slots, H, dim], [num_slots, H]
    const int32_t *slots;            // [n_seqs]
    const int32_t *cu;               // portions: [n_seqs + 1]; decode: null, row i is sequence i
    const int32_t *klen;             // tokens of every sequence, this step's included (decode: 0 = padded row)
    void *out;                       // [n, H vdim] dense
    int32_t n, n_seqs, heads, dim, vdim, num_slots;
    float q_scale, cap, eps;
};

constexpr float kMemoryGuard = 1e-6f;
constexpr float kNever = -1e30f;                           // a log weight of zero that may be added to and subtracted

// log gates of one row and head, in full fp32 whatever the tensors are
__device__ __forceinline__ void log_gates(const MlstmArgs &a, int64_t row, int head, float &in, float &keep) {
    const float zi = a.z[row * 2 * a.heads + head] + a.bias[head];
    const float zf = a.z[row * 2 * a.heads + a.heads + head] + a.bias[a.heads + head];
    in = a.cap * tanhf(zi / a.cap);
    const float f = a.cap * tanhf(zf / a.cap);
    keep = fminf(f, 0.f) - log1pf(expf(-fabsf(f)));
}

__device__ __forceinline__ float block_sum(float v, float *sh) {
    v = wave_sum(v);
    __syncthreads();
    if ((threadIdx.x & 63) == 0) sh[threadIdx.x >> 6] = v;
    __syncthreads();
    return (sh[0] + sh[1]) + (sh[2] + sh[3]);
}

// Any sizes, bf16 or fp32, portions and single tokens: one workgroup per (sequence, head) walks the
// tokens; the state stays in its slot (the L2 holds it) and is updated in place.
constexpr int kMemoryMaxDim = 512;

template <typename T>
__global__ __launch_bounds__(256) void mlstm_scan_any_kernel(MlstmArgs a) {
    __shared__ float sh_q[kMemoryMaxDim], sh_k[kMemoryMaxDim], sh_v[kMemoryMaxDim], sh_red[kMemoryMaxDim], sh_w[4];
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
    const int64_t cell = static_cast<int64_t>(slot) * a.heads + head;
    float *S = a.state + cell * a.dim * a.vdim, *N = a.mass + cell * a.dim;
    float m = start > 0 ? a.top[cell] : 0.f;
    int cols = 1;                                          // threads side by side over the value columns
    while (cols < a.vdim && cols < 256) cols <<= 1;
    const int groups = 256 / cols, c_lane = tid % cols, group = tid / cols;
    const int64_t qk = static_cast<int64_t>(a.heads) * a.dim;
    for (int t = 0; t < count; ++t) {
        const T *row = static_cast<const T *>(a.x) + static_cast<int64_t>(first + t) * a.stride;
        const T *q = row + static_cast<int64_t>(head) * a.dim, *k = q + qk;
        const T *v = row + 2 * qk + static_cast<int64_t>(head) * a.vdim, *gate = v + static_cast<int64_t>(a.heads) * a.vdim;
        float in, keep;
        log_gates(a, first + t, head, in, keep);
        const float m_new = fmaxf(keep + m, in);
        const float fk = expf(keep + m - m_new), fi = expf(in - m_new);
        m = m_new;
        const bool fresh = start == 0 && t == 0;
        float nq = 0.f;
        for (int i = tid; i < a.dim; i += 256) {
            const float qv = Elem<T>::to_f32(q[i]) * a.q_scale, kv = Elem<T>::to_f32(k[i]);
            sh_q[i] = qv;
            sh_k[i] = kv * fi;
            const float n = fmaf(fk, fresh ? 0.f : N[i], kv * fi);
            N[i] = n;
            nq = fmaf(n, qv, nq);
        }
        for (int c = tid; c < a.vdim; c += 256) sh_v[c] = Elem<T>::to_f32(v[c]);
        nq = block_sum(nq, sh_w);                          // (its barriers publish q, k and v)
        for (int c0 = 0; c0 < a.vdim; c0 += cols) {
            const int c = c0 + c_lane;
            float acc = 0.f;
            if (c < a.vdim) {
                const float vc = sh_v[c];
                for (int r = group; r < a.dim; r += groups) {
                    float *p = S + static_cast<int64_t>(r) * a.vdim + c;
                    const float s = fmaf(fk, fresh ? 0.f : *p, sh_k[r] * vc);
                    *p = s;
                    acc = fmaf(s, sh_q[r], acc);
                }
            }
            if (groups == 1) {
                if (c < a.vdim) sh_red[c] = acc;
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
        const float inv_den = 1.0f / (fmaxf(fabsf(nq), expf(-m)) + kMemoryGuard);
        float ss = 0.f;
        for (int c = tid; c < a.vdim; c += 256) { const float o = sh_red[c] * inv_den; ss = fmaf(o, o, ss); }
        const float inv = inv_den * rsqrtf(block_sum(ss, sh_w) / static_cast<float>(a.vdim) + a.eps);
        for (int c = tid; c < a.vdim; c += 256)
            out[(static_cast<int64_t>(first + t) * a.heads + head) * a.vdim + c] =
                Elem<T>::from_f32(sh_red[c] * inv * Elem<T>::to_f32(static_cast<const T *>(a.weight)[static_cast<int64_t>(head) * a.vdim + c]) *
                                  sigmoid_of<T>(Elem<T>::to_f32(gate[c])));
        __syncthreads();
    }
    if (tid == 0) a.top[cell] = m;
}

// Single tokens: one workgroup per (sequence, head) streams the state once -- read, scale, add k v^T, write,
// and the product with q on the way -- and finishes the head.  A thread owns four value columns (one 16-byte
// piece of a state row) of every kGroups-th row; eight rows are in flight at once.
// HBM: 2 * dim * (vdim + 1) * 4 bytes per (sequence, head).
template <typename T>
__global__ __launch_bounds__(256) void mlstm_step_kernel(MlstmArgs a) {
    __shared__ float sh_q[kMemoryMaxDim], sh_k[kMemoryMaxDim];
    __shared__ __align__(16) float sh_red[1024];
    __shared__ float sh_w[4], sh_n[4];
    const int seq = blockIdx.x / a.heads, head = blockIdx.x % a.heads;
    const int tid = threadIdx.x;
    const int start = a.klen[seq] - 1, slot = a.slots[seq];
    T *out = static_cast<T *>(a.out) + (static_cast<int64_t>(seq) * a.heads + head) * a.vdim;
    if (start < 0 || static_cast<uint32_t>(slot) >= static_cast<uint32_t>(a.num_slots)) {     // padded row
        for (int c = tid; c < a.vdim; c += 256) out[c] = Elem<T>::from_f32(0.f);
        return;
    }
    const int64_t cell = static_cast<int64_t>(slot) * a.heads + head;
    float *S = a.state + cell * a.dim * a.vdim, *N = a.mass + cell * a.dim;
    const int per_row = a.vdim / 4, groups = 256 / per_row;
    const int piece = tid % per_row, group = tid / per_row;
    const bool mine = group < groups;
    // the first rows of the state are on their way while the gates are formed
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
    const int64_t qk = static_cast<int64_t>(a.heads) * a.dim;
    const T *row = static_cast<const T *>(a.x) + static_cast<int64_t>(seq) * a.stride;
    const T *q = row + static_cast<int64_t>(head) * a.dim, *k = q + qk;
    const T *v = row + 2 * qk + static_cast<int64_t>(head) * a.vdim, *gate = v + static_cast<int64_t>(a.heads) * a.vdim;
    const float m_old = start > 0 ? a.top[cell] : 0.f;
    float in, keep;
    log_gates(a, seq, head, in, keep);
    const float m = fmaxf(keep + m_old, in);
    const float fk = expf(keep + m_old - m), fi = expf(in - m);
    float nq = 0.f;
    for (int i = tid; i < a.dim; i += 256) {
        const float qv = Elem<T>::to_f32(q[i]) * a.q_scale, kv = Elem<T>::to_f32(k[i]) * fi;
        sh_q[i] = qv;
        sh_k[i] = kv;
        const float n = fmaf(fk, start > 0 ? N[i] : 0.f, kv);
        N[i] = n;
        nq = fmaf(n, qv, nq);
    }
    nq = wave_sum(nq);
    if ((tid & 63) == 0) sh_n[tid >> 6] = nq;
    f32x4_t vv = {0.f, 0.f, 0.f, 0.f};
    if (mine)
#pragma unroll
        for (int i = 0; i < 4; ++i) vv[i] = Elem<T>::to_f32(v[4 * piece + i]);
    __syncthreads();
    if (tid == 0) a.top[cell] = m;                         // (every wavefront has read the old one)
    f32x4_t acc = {0.f, 0.f, 0.f, 0.f};
    for (int r0 = group; r0 < a.dim; r0 += kAhead * groups) {
#pragma unroll
        for (int i = 0; i < kAhead; ++i) {
            const int r = r0 + i * groups;
            if (mine && r < a.dim) {
                const float kr = sh_k[r], qr = sh_q[r];
#pragma unroll
                for (int j = 0; j < 4; ++j) {
                    s[i][j] = fmaf(fk, s[i][j], kr * vv[j]);
                    acc[j] = fmaf(s[i][j], qr, acc[j]);
                }
                __builtin_nontemporal_store(s[i], reinterpret_cast<f32x4_t *>(S + static_cast<int64_t>(r) * a.vdim) + piece);
            }
        }
        if (r0 + kAhead * groups < a.dim) fetch(r0 + kAhead * groups);
    }
    if (mine) *reinterpret_cast<f32x4_t *>(&sh_red[group * a.vdim + 4 * piece]) = acc;
    __syncthreads();
    const float inv_den = 1.0f / (fmaxf(fabsf((sh_n[0] + sh_n[1]) + (sh_n[2] + sh_n[3])), expf(-m)) + kMemoryGuard);
    float o[kMemoryMaxDim / 256], ss = 0.f;
#pragma unroll
    for (int i = 0; i < kMemoryMaxDim / 256; ++i) {
        const int c = tid + 256 * i;
        o[i] = 0.f;
        if (c < a.vdim)
            for (int g = 0; g < groups; ++g) o[i] += sh_red[g * a.vdim + c];
        o[i] *= inv_den;
        ss = fmaf(o[i], o[i], ss);
    }
    ss = wave_sum(ss);
    if ((tid & 63) == 0) sh_w[tid >> 6] = ss;
    __syncthreads();
    const float inv = rsqrtf(((sh_w[0] + sh_w[1]) + (sh_w[2] + sh_w[3])) / static_cast<float>(a.vdim) + a.eps);
#pragma unroll
    for (int i = 0; i < kMemoryMaxDim / 256; ++i) {
        const int c = tid + 256 * i;
        if (c < a.vdim)
            out[c] = Elem<T>::from_f32(o[i] * inv * Elem<T>::to_f32(static_cast<const T *>(a.weight)[static_cast<int64_t>(head) * a.vdim + c]) *
                                       sigmoid_of<T>(Elem<T>::to_f32(gate[c])));
    }
}

// ---- portions, bf16, on the matrix cores -----------------------------------------------------------
// A workgroup walks one (sequence, head) -- or one segment of it -- in chunks of 32 tokens.  With S, n, m the
// state before a chunk, b_t the sum of the log forget gates up to and including place t, a_s = i_s - b_s and
// M_t = max(m, max_{s <= t} a_s):
//     m_t = b_t + M_t
//     S_t^T q_t = e^{m - M_t} S^T q_t + sum_{s <= t} e^{a_s - M_t} (k_s . q_t) v_s       (n_t . q_t without v_s)
//     S' = e^{m - M_L} S + sum_s e^{a_s - M_L} k_s v_s^T                                 n', m' = b_L + M_L
// No exponent is positive.  q (its scale applied to the results), k and v are bf16 to begin with; what is
// fp32 -- weighted scores, the state, weighted v -- enters a product as the sum of two bf16 numbers.
// Wavefront w keeps its 16 NV value columns of S in accumulators, which are also the first operand of S^T q;
// n is one more column, repeated over a block of 16, whose rows the wavefronts share out.
// Long sequences are cut into segments so that the machine fills: the segments' own sums (kSums) are formed
// first, a scan over the segments turns them into the state each one starts from, then all run at once.
constexpr int kMemChunk = 32;
// token of a chunk that inner index 4 s + a of 16-lane group g stands for: groups whose LDS reads go together
// take every other token
__device__ __forceinline__ int memory_token(int g, int s, int a) { return 2 * (4 * (g & 1) + a) + (g >> 1) + 16 * s; }

struct MemorySegments {
    float *sums;         // [n_seqs, segments, H, pitch]: S, n, m of its own, sum of f, m at its start
    int32_t segments, length;
    int64_t pitch;
};

template <int DK, int NV, bool kSums>
__global__ __launch_bounds__(256, DK * NV > 256 ? 1 : 2) void mlstm_chunk_kernel(const MlstmArgs a, const MemorySegments sg) {
    constexpr int kC = kMemChunk, kDB = DK / 16, kPitch = DK * 2 + 16, kVW = 64 * NV, kVPitch = kVW * 2 + 16, kPPitch = kC * 2 + 16;
    constexpr int kQ = 0, kK = kSums ? 0 : kC * kPitch, kV = kK + kC * kPitch, kP = kV + kC * kVPitch;
    constexpr int kPieces = DK / 64, kMS = (DK / 32 + 3) / 4;
    __shared__ __attribute__((aligned(16))) unsigned char smem[kP + (kSums ? 0 : 2 * kC * kPPitch)];
    __shared__ float sh_ss[4][kC], sh_nq[4][kC], sh_rs[2][kC];
    __shared__ float sh_a[kC], sh_M[kC], sh_g[kC], sh_floor[kC], sh_end[2];
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
    const int64_t cell = static_cast<int64_t>(have_slot ? slot : 0) * a.heads + head;
    float *seg_state = sg.sums + ((static_cast<int64_t>(seq) * sg.segments + seg) * a.heads + head) * sg.pitch;
    const int v0 = wave * 16 * NV;                       // this wavefront's first value column

    f32x4_t S[kDB][NV], N[kMS][2];
    float m0 = kSums ? kNever : 0.f, f_sum = 0.f;        // (of wavefront 3, which forms the weights)
    {
        const bool carried = !kSums && (sg.segments > 1 || (have_slot && start > 0));
        const float *src = sg.segments > 1 ? seg_state : a.state + cell * state_size;
        const float *nsrc = sg.segments > 1 ? seg_state + state_size : a.mass + cell * a.dim;
        if (carried) m0 = sg.segments > 1 ? seg_state[state_size + a.dim + 2] : a.top[cell];
#pragma unroll
        for (int db = 0; db < kDB; ++db)
#pragma unroll
            for (int vb = 0; vb < NV; ++vb)
#pragma unroll
                for (int i = 0; i < 4; ++i) {
                    const int d = 16 * db + 4 * g + i, v = v0 + 16 * vb + r;
                    S[db][vb][i] = carried && d < a.dim && v < a.vdim ? src[static_cast<int64_t>(d) * a.vdim + v] : 0.f;
                }
#pragma unroll
        for (int x = 0; x < kMS; ++x)
#pragma unroll
            for (int h = 0; h < 2; ++h)
#pragma unroll
                for (int i = 0; i < 4; ++i) {
                    const int d = 32 * (wave + 4 * x) + 16 * h + 4 * g + i;
                    N[x][h][i] = carried && d < a.dim ? nsrc[d] : 0.f;
                }
    }
    const int s_qb = wave >> 1, s_kb = wave & 1;         // the block of scores this wavefront computes
    const float inv_vdim = 1.0f / static_cast<float>(a.vdim);
    constexpr float kLog2e = 1.4426950408889634f;

    const int64_t qk = static_cast<int64_t>(a.heads) * a.dim;
    const bf16_t *xq = static_cast<const bf16_t *>(a.x) + static_cast<int64_t>(head) * a.dim;
    const bf16_t *xv = static_cast<const bf16_t *>(a.x) + 2 * qk + static_cast<int64_t>(head) * a.vdim;
    const bf16_t *xg = xv + static_cast<int64_t>(a.heads) * a.vdim;
    // a thread's pieces of q, k and v (32 rows) are loaded one chunk ahead
    u32x4_t rq[kSums ? 1 : kPieces], rk[kPieces], rv[NV];
    auto fetch = [&](int t0) __attribute__((always_inline)) {
#pragma unroll
        for (int i = 0; i < kPieces; ++i) {
            const int p = i * 256 + tid, row = p / (DK / 8), e = p % (DK / 8) * 8;
            const bool in = t0 + row < t_end && e < a.dim;
            const bf16_t *x = xq + static_cast<int64_t>(first + t0 + row) * a.stride + e;
            if (!kSums) { rq[kSums ? 0 : i] = u32x4_t{0, 0, 0, 0}; if (in) rq[kSums ? 0 : i] = *reinterpret_cast<const u32x4_t *>(x); }
            rk[i] = u32x4_t{0, 0, 0, 0};
            if (in) rk[i] = *reinterpret_cast<const u32x4_t *>(x + qk);
        }
#pragma unroll
        for (int i = 0; i < NV; ++i) {
            const int p = i * 256 + tid, row = p / (kVW / 8), e = p % (kVW / 8) * 8;
            rv[i] = u32x4_t{0, 0, 0, 0};
            if (t0 + row < t_end && e < a.vdim) rv[i] = *reinterpret_cast<const u32x4_t *>(xv + static_cast<int64_t>(first + t0 + row) * a.stride + e);
        }
    };
    // log gates of the chunk: lane t (and t + 32) of wavefront 3 holds place t
    float pre_b = 0.f, pre_a = kNever, pre_max = kNever;
    auto gates = [&](int t0) __attribute__((always_inline)) {
        if (wave != 3) return;
        const int t = lane & 31;
        float in = kNever, keep = 0.f;
        if (t0 + t < t_end) log_gates(a, first + t0 + t, head, in, keep);
        pre_b = keep;
#pragma unroll
        for (int d = 1; d < 32; d <<= 1) {
            const float o = __shfl_up(pre_b, d, 32);
            if (t >= d) pre_b += o;
        }
        pre_a = in - pre_b;
        pre_max = pre_a;
#pragma unroll
        for (int d = 1; d < 32; d <<= 1) {
            const float o = __shfl_up(pre_max, d, 32);
            if (t >= d) pre_max = fmaxf(pre_max, o);
        }
    };
    fetch(t_begin);
    gates(t_begin);

    for (int t0 = t_begin; t0 < t_end; t0 += kC) {
        const int L = min(kC, t_end - t0);
        // ---- q, k, v and the weights of the chunk into LDS ------------------------------------------
#pragma unroll
        for (int i = 0; i < kPieces; ++i) {
            const int p = i * 256 + tid, at = p / (DK / 8) * kPitch + p % (DK / 8) * 16;
            if (!kSums) *(lds_u32x4_ptr)(lds + kQ + at) = rq[kSums ? 0 : i];
            *(lds_u32x4_ptr)(lds + kK + at) = rk[i];
        }
#pragma unroll
        for (int i = 0; i < NV; ++i) {
            const int p = i * 256 + tid;
            *(lds_u32x4_ptr)(lds + kV + p / (kVW / 8) * kVPitch + p % (kVW / 8) * 16) = rv[i];
        }
        if (wave == 3) {
            const float M = fmaxf(m0, pre_max), m = pre_b + M;
            if (lane < kC) {
                sh_a[lane] = pre_a * kLog2e;
                sh_M[lane] = M * kLog2e;
                sh_g[lane] = __builtin_amdgcn_exp2f((m0 - M) * kLog2e) * a.q_scale;
                sh_floor[lane] = __builtin_amdgcn_exp2f(-m * kLog2e);
            }
            const float M_end = __shfl(M, L - 1, 64), b_end = __shfl(pre_b, L - 1, 64);
            if (lane == 0) {
                sh_end[0] = M_end * kLog2e;
                sh_end[1] = __builtin_amdgcn_exp2f((m0 - M_end) * kLog2e);
            }
            m0 = b_end + M_end;
            f_sum += b_end;
        }
        __syncthreads();
        if (t0 + kC < t_end) fetch(t0 + kC);
        const float M_end = sh_end[0], g_chunk = sh_end[1];
        float vfac[8];
#pragma unroll
        for (int e = 0; e < 8; ++e) vfac[e] = __builtin_amdgcn_exp2f(sh_a[memory_token(g, e >> 2, e & 3)] - M_end);
        f32x4_t O[NV][2];
        if (!kSums) {
            // operands in the accumulators' inner order: 32 ks + 4 g + [0, 4) and 16 further on
            auto row_frag = [&](int at, int row, int ks) __attribute__((always_inline)) -> u32x4_t {
                typedef __attribute__((address_space(3))) u32x2_t *lds_u32x2_ptr;
                const lds_char_ptr p = lds + at + row * kPitch + 64 * ks + 8 * g;
                const u32x2_t x = *(lds_u32x2_ptr)p, y = *(lds_u32x2_ptr)(p + 32);
                return u32x4_t{x[0], x[1], y[0], y[1]};
            };
            f32x4_t on[2];
            on[0] = on[1] = f32x4_t{0.f, 0.f, 0.f, 0.f};
#pragma unroll
            for (int vb = 0; vb < NV; ++vb) O[vb][0] = O[vb][1] = f32x4_t{0.f, 0.f, 0.f, 0.f};
            f32x4_t sc = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
            for (int ks = 0; ks < DK / 32; ++ks) {
                u32x4_t qf[2];
#pragma unroll
                for (int qb = 0; qb < 2; ++qb) qf[qb] = row_frag(kQ, 16 * qb + r, ks);
                if (s_qb >= s_kb) sc = mfma16(row_frag(kK, 16 * s_kb + r, ks), s_qb ? qf[1] : qf[0], sc);     // (wave-uniform)
                u32x4_t hi, lo;
#pragma unroll
                for (int vb = 0; vb < NV; ++vb) {
                    const float f[8] = {S[2 * ks][vb][0], S[2 * ks][vb][1], S[2 * ks][vb][2], S[2 * ks][vb][3],
                                        S[2 * ks + 1][vb][0], S[2 * ks + 1][vb][1], S[2 * ks + 1][vb][2], S[2 * ks + 1][vb][3]};
                    split8(f, hi, lo);
#pragma unroll
                    for (int qb = 0; qb < 2; ++qb) {
                        O[vb][qb] = mfma16(hi, qf[qb], O[vb][qb]);
                        O[vb][qb] = mfma16(lo, qf[qb], O[vb][qb]);
                    }
                }
                if (ks % 4 == wave) {                    // (wave-uniform)
                    const f32x4_t &n0 = N[ks / 4][0], &n1 = N[ks / 4][1];
                    const float f[8] = {n0[0], n0[1], n0[2], n0[3], n1[0], n1[1], n1[2], n1[3]};
                    split8(f, hi, lo);
#pragma unroll
                    for (int qb = 0; qb < 2; ++qb) {
                        on[qb] = mfma16(hi, qf[qb], on[qb]);
                        on[qb] = mfma16(lo, qf[qb], on[qb]);
                    }
                }
            }
#pragma unroll
            for (int qb = 0; qb < 2; ++qb) {
                const float gq = sh_g[16 * qb + r];
#pragma unroll
                for (int vb = 0; vb < NV; ++vb)
#pragma unroll
                    for (int i = 0; i < 4; ++i) O[vb][qb][i] *= gq;
                if (g == 0) sh_nq[wave][16 * qb + r] = on[qb][0] * gq;
            }
            // weighted scores to LDS: row = query, columns in memory_token order.  Keys 4 g .. 4 g + 3 of block
            // s_kb: the even two are neighbours there, and so are the odd two, 16 columns on
            const int qrow = 16 * s_qb + r;
            const float Mq = sh_M[qrow];
            float p4[4], rs = 0.f;
#pragma unroll
            for (int i = 0; i < 4; ++i) {
                const int key = 16 * s_kb + 4 * g + i;
                p4[i] = key <= qrow ? sc[i] * a.q_scale * __builtin_amdgcn_exp2f(sh_a[key] - Mq) : 0.f;
                rs += p4[i];
            }
            rs += __shfl_xor(rs, 16, 64);
            rs += __shfl_xor(rs, 32, 64);
            if (g == 0) sh_rs[s_kb][qrow] = rs;
            uint32_t he, le, ho, lo;
            split_pair(p4[0], p4[2], he, le);
            split_pair(p4[1], p4[3], ho, lo);
            typedef __attribute__((address_space(3))) uint32_t *lds_u32_ptr;
            const lds_char_ptr p = lds + kP + qrow * kPPitch + 2 * (8 * (g >> 1) + 4 * s_kb + 2 * (g & 1));
            *(lds_u32_ptr)p = he;
            *(lds_u32_ptr)(p + 32) = ho;
            *(lds_u32_ptr)(p + kC * kPPitch) = le;
            *(lds_u32_ptr)(p + kC * kPPitch + 32) = lo;
            __syncthreads();
        }
        // ---- v^T fragments: the second product's first operand and, weighted, the state's second ------
        auto token_frag = [&](int at, int pitch, int col) __attribute__((always_inline)) -> u32x4_t {
            const lds_char_ptr p = lds + at + memory_token(g, 0, r >> 2) * pitch + 2 * (col + 4 * (r & 3));
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
        u32x4_t vh[NV], vl[NV], oh, ol;
        split8(vfac, oh, ol);
#pragma unroll
        for (int vb = 0; vb < NV; ++vb) {
            float f[8];
            unpack8(make_uint4(vf[vb][0], vf[vb][1], vf[vb][2], vf[vb][3]), f);
#pragma unroll
            for (int e = 0; e < 8; ++e) f[e] *= vfac[e];
            split8(f, vh[vb], vl[vb]);
        }
        // what the end of this chunk and the start of the next one wait for: gates
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
        if (t0 + kC < t_end) gates(t0 + kC);
#pragma unroll
        for (int db = 0; db < kDB; ++db) {
            const u32x4_t kf = token_frag(kK, kPitch, 16 * db);
#pragma unroll
            for (int vb = 0; vb < NV; ++vb) {
#pragma unroll
                for (int i = 0; i < 4; ++i) S[db][vb][i] *= g_chunk;
                S[db][vb] = mfma16(kf, vh[vb], S[db][vb]);
                S[db][vb] = mfma16(kf, vl[vb], S[db][vb]);
            }
            if (db / 2 % 4 == wave) {                    // (wave-uniform)
                f32x4_t &n = N[db / 8][db & 1];
#pragma unroll
                for (int i = 0; i < 4; ++i) n[i] *= g_chunk;
                n = mfma16(kf, oh, n);
                n = mfma16(kf, ol, n);
            }
        }
        float inv_den[2], floor_q[2];
        if (!kSums) {
            // ---- denominator and head norm (value columns are spread over registers, lane groups and wavefronts)
#pragma unroll
            for (int qb = 0; qb < 2; ++qb) {
                const int row = 16 * qb + r;
                floor_q[qb] = sh_floor[row];
                const float nq = (sh_nq[0][row] + sh_nq[1][row]) + (sh_nq[2][row] + sh_nq[3][row]) + (sh_rs[0][row] + sh_rs[1][row]);
                inv_den[qb] = 1.0f / (fmaxf(fabsf(nq), floor_q[qb]) + kMemoryGuard);
                float ss = 0.f;
#pragma unroll
                for (int vb = 0; vb < NV; ++vb)
#pragma unroll
                    for (int i = 0; i < 4; ++i) { const float o = O[vb][qb][i] * inv_den[qb]; ss = fmaf(o, o, ss); }
                ss += __shfl_xor(ss, 16, 64);
                ss += __shfl_xor(ss, 32, 64);
                if (g == 0) sh_ss[wave][row] = ss;
            }
        }
        __syncthreads();
        if (!kSums) {
#pragma unroll
            for (int qb = 0; qb < 2; ++qb) {
                const int row = 16 * qb + r;
                const float ss = (sh_ss[0][row] + sh_ss[1][row]) + (sh_ss[2][row] + sh_ss[3][row]);
                const float inv = inv_den[qb] * rsqrtf(fmaf(ss, inv_vdim, a.eps));
                if (row >= L) continue;
                const int64_t t = first + t0 + row;
                bf16_t *out = static_cast<bf16_t *>(a.out) + (t * a.heads + head) * a.vdim;
                const bf16_t *weight = static_cast<const bf16_t *>(a.weight) + static_cast<int64_t>(head) * a.vdim;
#pragma unroll
                for (int vb = 0; vb < NV; ++vb) {
                    const int v = v0 + 16 * vb + 4 * g;
                    if (v < a.vdim) {
                        const u32x2_t z = gate[qb][vb], w = *reinterpret_cast<const u32x2_t *>(weight + v);
                        const float zf[4] = {bf16lo_to_f32(z[0]), bf16hi_to_f32(z[0]), bf16lo_to_f32(z[1]), bf16hi_to_f32(z[1])};
                        const float wf[4] = {bf16lo_to_f32(w[0]), bf16hi_to_f32(w[0]), bf16lo_to_f32(w[1]), bf16hi_to_f32(w[1])};
                        float y[4];
#pragma unroll
                        for (int i = 0; i < 4; ++i) y[i] = O[vb][qb][i] * inv * wf[i] * sigmoid_of<bf16_t>(zf[i]);
                        *reinterpret_cast<u32x2_t *>(out + v) = u32x2_t{pack_bf16x2(y[0], y[1]), pack_bf16x2(y[2], y[3])};
                    }
                }
            }
        }
    }
    if (!kSums && (t_end < count || !have_slot)) return;
    float *dst = kSums ? seg_state : a.state + cell * state_size;
    float *ndst = kSums ? seg_state + state_size : a.mass + cell * a.dim;
#pragma unroll
    for (int db = 0; db < kDB; ++db)
#pragma unroll
        for (int vb = 0; vb < NV; ++vb)
#pragma unroll
            for (int i = 0; i < 4; ++i) {
                const int d = 16 * db + 4 * g + i, v = v0 + 16 * vb + r;
                if (d < a.dim && v < a.vdim) dst[static_cast<int64_t>(d) * a.vdim + v] = S[db][vb][i];
            }
    if (r == 0)
#pragma unroll
        for (int x = 0; x < kMS; ++x)
#pragma unroll
            for (int h = 0; h < 2; ++h)
#pragma unroll
                for (int i = 0; i < 4; ++i) {
                    const int ks = wave + 4 * x, d = 32 * ks + 16 * h + 4 * g + i;
                    if (ks < DK / 32 && d < a.dim) ndst[d] = N[x][h][i];
                }
    if (wave == 3 && lane == 0) {
        if (kSums) {
            seg_state[state_size + a.dim] = m0;
            seg_state[state_size + a.dim + 1] = f_sum;
        } else {
            a.top[cell] = m0;
        }
    }
}

// Replaces every segment's own sums by the state the segment starts from; one thread per four elements of
// (S, n) (both sizes are multiples of 8).
__global__ __launch_bounds__(256) void mlstm_segment_scan_kernel(const MlstmArgs a, const MemorySegments sg) {
    const int head = blockIdx.x % a.heads, seq = blockIdx.x / a.heads;
    const int64_t size = static_cast<int64_t>(a.dim) * a.vdim, all = size + a.dim;
    const int64_t e = (static_cast<int64_t>(blockIdx.y) * 256 + threadIdx.x) * 4;
    const int count = a.cu[seq + 1] - a.cu[seq], start = a.klen[seq] - count;
    if (e >= all || count <= 0 || start < 0) return;
    const int slot = a.slots[seq];
    const bool carried = start > 0 && static_cast<uint32_t>(slot) < static_cast<uint32_t>(a.num_slots);
    const int64_t cell = static_cast<int64_t>(carried ? slot : 0) * a.heads + head;
    f32x4_t run = {0.f, 0.f, 0.f, 0.f};
    if (carried) run = *reinterpret_cast<const f32x4_t *>(e < size ? a.state + cell * size + e : a.mass + cell * a.dim + (e - size));
    float m = carried ? a.top[cell] : 0.f;
    const int segments = min(sg.segments, (count - 1) / sg.length + 1);
    float *base = sg.sums + (static_cast<int64_t>(seq) * sg.segments * a.heads + head) * sg.pitch;
    const int64_t step = static_cast<int64_t>(a.heads) * sg.pitch;
    constexpr int kAhead = 16;                            // loads in flight together
    for (int s0 = 0; s0 < segments; s0 += kAhead) {
        f32x4_t own[kAhead];
        float own_m[kAhead], own_f[kAhead];
#pragma unroll
        for (int i = 0; i < kAhead; ++i) {
            own[i] = f32x4_t{0.f, 0.f, 0.f, 0.f};
            own_m[i] = kNever;
            own_f[i] = 0.f;
            if (s0 + i + 1 < segments) {
                const float *p = base + (s0 + i) * step;
                own[i] = *reinterpret_cast<const f32x4_t *>(p + e);
                own_m[i] = p[all];
                own_f[i] = p[all + 1];
            }
        }
#pragma unroll
        for (int i = 0; i < kAhead; ++i)
            if (s0 + i < segments) {
                float *p = base + (s0 + i) * step;
                *reinterpret_cast<f32x4_t *>(p + e) = run;
                if (e == 0) p[all + 2] = m;
                const float m_new = fmaxf(own_f[i] + m, own_m[i]);
                const float keep = expf(own_f[i] + m - m_new), take = expf(own_m[i] - m_new);
                m = m_new;
#pragma unroll
                for (int j = 0; j < 4; ++j) run[j] = fmaf(keep, run[j], take * own[i][j]);
            }
    }
}

// Segments of a call: enough (sequence, head, segment) workgroups for the machine, none shorter than 256
// tokens.  Depends on shapes only.
static MemorySegments plan_memory(int32_t n_seqs, int32_t heads, int32_t dim, int32_t vdim, int32_t max_q) {
    MemorySegments sg{};
    const int64_t walks = std::max<int64_t>(1, static_cast<int64_t>(n_seqs) * heads);
    const int64_t want = std::min<int64_t>(std::max<int64_t>(1, 512 / walks), std::max(1, max_q / 256));
    const int64_t length = (max_q + want - 1) / want;
    sg.length = static_cast<int32_t>(std::max<int64_t>(kMemChunk, (length + kMemChunk - 1) / kMemChunk * kMemChunk));
    sg.segments = std::max(1, (max_q + sg.length - 1) / sg.length);
    sg.pitch = static_cast<int64_t>(dim) * vdim + dim + 4;
    return sg;
}

template <int DK, int NV>
static int launch_memory(const MlstmArgs &a, const MemorySegments &sg, hipStream_t s) {
    const dim3 grid(static_cast<uint32_t>(a.n_seqs) * sg.segments * a.heads), block(256);
    if (sg.segments > 1) {
        hipLaunchKernelGGL((mlstm_chunk_kernel<DK, NV, true>), grid, block, 0, s, a, sg);
        int rc = launch_status();
        if (rc != NVA_OK) return rc;
        hipLaunchKernelGGL(mlstm_segment_scan_kernel, dim3(a.n_seqs * a.heads, (a.dim * (a.vdim + 1) + 1023) / 1024), block, 0, s, a, sg);
        rc = launch_status();
        if (rc != NVA_OK) return rc;
    }
    hipLaunchKernelGGL((mlstm_chunk_kernel<DK, NV, false>), grid, block, 0, s, a, sg);
    return launch_status();
}

// Sizes the chunked form is built for: everything vectors can hold with the state in registers.
static bool memory_chunks_ok(int32_t dim, int32_t vdim) {
    return dim % 8 == 0 && vdim % 8 == 0 && ((dim <= 128 && vdim <= 256) || (dim <= 256 && vdim <= 128));
}

template <int DK>
static int launch_memory_dk(const MlstmArgs &a, const MemorySegments &sg, hipStream_t s) {
    if (a.vdim <= 64) return launch_memory<DK, 1>(a, sg, s);
    if (a.vdim <= 128) return launch_memory<DK, 2>(a, sg, s);
    if constexpr (DK <= 128) return launch_memory<DK, 4>(a, sg, s);
    return NVA_ERR_UNSUPPORTED_GEOMETRY;
}

}  // namespace nva

extern "C" size_t nva_mlstm_workspace_bytes(int32_t n_seqs, int32_t max_seqlen_q, int32_t num_heads, int32_t qk_dim,
                                            int32_t v_dim, int32_t dtype) {
    if (n_seqs <= 0 || max_seqlen_q <= 0 || num_heads <= 0 || qk_dim <= 0 || v_dim <= 0) return 0;
    if (dtype != NVA_DTYPE_BF16 || !nva::memory_chunks_ok(qk_dim, v_dim)) return 0;
    const nva::MemorySegments sg = nva::plan_memory(n_seqs, num_heads, qk_dim, v_dim, max_seqlen_q);
    if (sg.segments == 1) return 0;
    return static_cast<size_t>(n_seqs) * sg.segments * num_heads * sg.pitch * sizeof(float);
}

extern "C" int nva_mlstm(const void *qkvg, int64_t row_stride, const float *gate_logits, const float *gate_bias,
                         const void *norm_weight, float *state, float *mass, float *top, const int32_t *state_slots_of_seq,
                         const int32_t *cu_seqlens_q, const int32_t *seq_lens, void *out, void *workspace,
                         size_t workspace_bytes, int32_t n_tokens, int32_t n_seqs, int32_t max_seqlen_q, int32_t num_heads,
                         int32_t qk_dim, int32_t v_dim, int32_t num_state_slots, float q_scale, float gate_cap, float eps,
                         int32_t dtype, void *stream) {
    using namespace nva;
    if (n_tokens < 0 || n_seqs < 0 || max_seqlen_q < 0 || num_heads <= 0 || qk_dim <= 0 || v_dim <= 0 || num_state_slots < 0 || !(gate_cap > 0.f))
        return NVA_ERR_BAD_SHAPE;
    if (qk_dim > kMemoryMaxDim || v_dim > kMemoryMaxDim || !known_dtype(dtype)) return NVA_ERR_UNSUPPORTED_GEOMETRY;
    if (n_tokens == 0 || n_seqs == 0) return NVA_OK;
    if (!qkvg || !gate_logits || !gate_bias || !norm_weight || !state || !mass || !top || !state_slots_of_seq || !seq_lens || !out)
        return NVA_ERR_NULL_POINTER;
    if (cu_seqlens_q == nullptr && n_seqs != n_tokens) return NVA_ERR_BAD_SHAPE;
    if (row_stride < 2 * static_cast<int64_t>(num_heads) * (qk_dim + v_dim)) return NVA_ERR_BAD_STRIDE;
    if (static_cast<int64_t>(n_seqs) * num_heads > 0x7fffffffLL) return NVA_ERR_BAD_SHAPE;
    MlstmArgs a{};
    a.x = qkvg; a.stride = row_stride; a.z = gate_logits; a.bias = gate_bias; a.weight = norm_weight; a.state = state; a.mass = mass;
    a.top = top; a.slots = state_slots_of_seq; a.cu = cu_seqlens_q; a.klen = seq_lens; a.out = out; a.n = n_tokens; a.n_seqs = n_seqs;
    a.heads = num_heads; a.dim = qk_dim; a.vdim = v_dim; a.num_slots = num_state_slots; a.q_scale = q_scale; a.cap = gate_cap; a.eps = eps;
    hipStream_t s = static_cast<hipStream_t>(stream);
    const dim3 grid(static_cast<uint32_t>(n_seqs) * num_heads), block(256);
    if (cu_seqlens_q == nullptr && v_dim % 4 == 0 && aligned16(state)) {
        if (dtype == NVA_DTYPE_BF16) hipLaunchKernelGGL((mlstm_step_kernel<bf16_t>), grid, block, 0, s, a);
        else hipLaunchKernelGGL((mlstm_step_kernel<float>), grid, block, 0, s, a);
        return launch_status();
    }
    if (cu_seqlens_q != nullptr && dtype == NVA_DTYPE_BF16 && memory_chunks_ok(qk_dim, v_dim) && row_stride % 8 == 0 &&
        aligned16(state) && aligned16(mass) && aligned16(qkvg) && aligned16(out) && aligned16(norm_weight)) {
        MemorySegments sg = plan_memory(n_seqs, num_heads, qk_dim, v_dim, max_seqlen_q);
        sg.sums = static_cast<float *>(workspace);
        if (sg.segments > 1) {
            if (!workspace) return NVA_ERR_NULL_POINTER;
            if (!aligned16(workspace)) return NVA_ERR_MISALIGNED;
            if (workspace_bytes < nva_mlstm_workspace_bytes(n_seqs, max_seqlen_q, num_heads, qk_dim, v_dim, dtype))
                return NVA_ERR_WORKSPACE_TOO_SMALL;
        }
        if (static_cast<int64_t>(n_seqs) * sg.segments * num_heads > 0x7fffffffLL) return NVA_ERR_BAD_SHAPE;
        if (qk_dim <= 64) return launch_memory_dk<64>(a, sg, s);
        if (qk_dim <= 128) return launch_memory_dk<128>(a, sg, s);
        return launch_memory_dk<256>(a, sg, s);
    }
    if (dtype == NVA_DTYPE_BF16) hipLaunchKernelGGL((mlstm_scan_any_kernel<bf16_t>), grid, block, 0, s, a);
    else hipLaunchKernelGGL((mlstm_scan_any_kernel<float>), grid, block, 0, s, a);
    return launch_status();
}
