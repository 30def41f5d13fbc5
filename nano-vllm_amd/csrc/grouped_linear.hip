// Matrix products whose weights come in groups, and the router that assigns rows to them.
//   dense groups   out[r, g] = W_g x[r, g] for every row r and group g (per-head products; one group: a plain
//                  product with few outputs, in fp32 where asked for)
//   routed groups  out[p] = W_e x[p / terms] for every assignment p = row * terms + k of a row to an expert e;
//                  lists[e] holds the assignments of expert e in any order, counts[e] their number
//   gated          W has 2 n_out rows (gate | up): out = g sigmoid(slope g) (u + shift), g = min(gate, limit), u = clamp(up, limit)
//                  (slope 1, shift 0, no limit: silu(gate) * up)
//                  (routed: an assignment's weight may belong to what its expert reads; it then multiplies gate and up)
//   squared relu   of a dense group's results, where asked for
//   router         logits (with a bias) in fp32, the best `terms`, their weights (from a softmax over all experts, normalised, or
//                  their sigmoids as they are), lists;
//                  and the sigmoids of further outputs, gates of what every row runs
// bf16 tensors go through the matrix cores, fp32 ones and odd sizes through plain fp32 kernels.
#include "nva_elem.h"
#include "nva_matrix.h"

#include <math.h>

#include <algorithm>
#include <type_traits>

namespace nva {

struct GateForm {
    float limit, slope, shift;
};

struct LinearArgs {
    const void *x;
    int64_t x_stride, x_group;       // elements between rows, between groups (dense)
    const void *w;                   // [groups][n_out or 2 n_out][k]
    void *out;
    int64_t o_stride, o_group;
    const int32_t *lists, *counts;   // routed: [groups, list_stride], [groups]
    int64_t list_stride;
    int32_t rows, groups, n_out, k;  // rows: dense rows, or assignments in all
    int32_t x_div;                   // routed: x row = assignment / x_div
    GateForm gate;                   // gated
    int32_t squared_relu;            // of the results (not gated)
    const float *in_weight;          // gated, routed: of assignment p at p / terms * in_stride + p % terms, or null
    int64_t in_stride;
    int32_t terms;
};

// what the rows a group reads are multiplied by
__device__ __forceinline__ float input_weight(const LinearArgs &a, int row) {
    return a.in_weight == nullptr ? 1.0f : a.in_weight[row / a.terms * a.in_stride + row % a.terms];
}

// number of rows of a group, and where its i-th row comes from and goes to
__device__ __forceinline__ int group_rows(const LinearArgs &a, int g) {
    return a.lists == nullptr ? a.rows : min(max(a.counts[g], 0), static_cast<int32_t>(a.list_stride));
}
__device__ __forceinline__ int group_row(const LinearArgs &a, int g, int i) {
    return a.lists == nullptr ? i : min(max(a.lists[g * a.list_stride + i], 0), a.rows - 1);
}
__device__ __forceinline__ int64_t x_offset(const LinearArgs &a, int g, int row) {
    return a.lists == nullptr ? row * a.x_stride + g * a.x_group : row / a.x_div * a.x_stride;
}
__device__ __forceinline__ int64_t out_offset(const LinearArgs &a, int g, int row) {
    return row * a.o_stride + (a.lists == nullptr ? g * a.o_group : 0);
}

template <typename T> __device__ __forceinline__ float gated_value(const GateForm &f, float gate, float up) {
    const float g = fminf(gate, f.limit), u = fminf(fmaxf(up, -f.limit), f.limit);
    return g * sigmoid_of<T>(f.slope * g) * (u + f.shift);
}
__device__ __forceinline__ float result_of(const LinearArgs &a, float v) {
    if (!a.squared_relu) return v;
    v = fmaxf(v, 0.f);
    return v * v;
}

// ---- any sizes, bf16 or fp32: tiles of 16 rows x 64 outputs in plain fp32 arithmetic ----------------
template <typename T, typename O, bool kGated>
__global__ __launch_bounds__(256) void linear_any_kernel(LinearArgs a) {
    constexpr int kParts = kGated ? 2 : 1, kK = 32;
    __shared__ float sx[16][kK + 1], sw[kParts][64][kK + 1];
    const int g = blockIdx.y, n0 = blockIdx.x * 64, tid = threadIdx.x;
    const int r = tid >> 4, c = tid & 15;
    const int count = group_rows(a, g);
    const T *w = static_cast<const T *>(a.w) + static_cast<int64_t>(g) * kParts * a.n_out * a.k;
    for (int m0 = blockIdx.z * 16; m0 < count; m0 += gridDim.z * 16) {
        float acc[kParts][4];
#pragma unroll
        for (int p = 0; p < kParts; ++p)
#pragma unroll
            for (int j = 0; j < 4; ++j) acc[p][j] = 0.f;
        const int row = group_row(a, g, min(m0 + r, count - 1));
        const T *x = static_cast<const T *>(a.x) + x_offset(a, g, row);
        for (int k0 = 0; k0 < a.k; k0 += kK) {
            for (int i = c; i < kK; i += 16) sx[r][i] = k0 + i < a.k ? Elem<T>::to_f32(x[k0 + i]) : 0.f;
            for (int i = tid; i < kParts * 64 * kK; i += 256) {
                const int kk = i % kK, n = i / kK % 64, p = i / kK / 64;
                sw[p][n][kk] = k0 + kk < a.k && n0 + n < a.n_out ? Elem<T>::to_f32(w[(static_cast<int64_t>(p) * a.n_out + n0 + n) * a.k + k0 + kk]) : 0.f;
            }
            __syncthreads();
#pragma unroll 8
            for (int kk = 0; kk < kK; ++kk)
#pragma unroll
                for (int p = 0; p < kParts; ++p)
#pragma unroll
                    for (int j = 0; j < 4; ++j) acc[p][j] = fmaf(sx[r][kk], sw[p][c + 16 * j][kk], acc[p][j]);
            __syncthreads();
        }
        if (m0 + r < count) {
            O *out = static_cast<O *>(a.out) + out_offset(a, g, row);
            const float f = kGated ? input_weight(a, row) : 1.0f;
#pragma unroll
            for (int j = 0; j < 4; ++j) {
                const int n = n0 + c + 16 * j;
                if (n < a.n_out) out[n] = Elem<O>::from_f32(kGated ? gated_value<T>(a.gate, f * acc[0][j], f * acc[kParts - 1][j]) : result_of(a, acc[0][j]));
            }
        }
    }
}

// ---- bf16, few rows per group: the weights are streamed once per 16 MT rows ------------------------
// A workgroup takes 16 NB outputs of a group (NB blocks of 16 gates and the 16 ups that belong to them), its four
// wavefronts a quarter of the inner dimension each, weights and rows straight from memory into operands
// (weights first operand: an accumulator holds four consecutive outputs of one row).  The quarters meet in LDS.
// Groups from all.groups on are those of `beside`: other, dense products of the same kind in the same launch.
template <int MT, int NB, bool kGated, typename O>
__global__ __launch_bounds__(256) void linear_skinny_kernel(const LinearArgs all, const LinearArgs beside) {
    constexpr int kParts = kGated ? 2 : 1, kBlocks = kParts * NB, kAhead = MT * NB == 1 ? 8 : 4;
    __shared__ __attribute__((aligned(16))) float part[4][MT * 16][kBlocks * 16 + 4];
    const bool first = static_cast<int>(blockIdx.y) < all.groups;
    const LinearArgs &a = first ? all : beside;
    const int g = first ? blockIdx.y : blockIdx.y - all.groups, n0 = blockIdx.x * 16 * NB;
    if (n0 >= a.n_out) return;                           // (the grid is as wide as the wider of the two)
    const int tid = threadIdx.x, lane = tid & 63, r = lane & 15, q = lane >> 4;
    const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
    const int count = group_rows(a, g);
    const int steps = (a.k + 31) / 32, per_wave = (steps + 3) / 4;
    const int s_begin = wave * per_wave, s_end = min(steps, s_begin + per_wave);
    const bf16_t *w[kBlocks];
#pragma unroll
    for (int b = 0; b < kBlocks; ++b)
        w[b] = static_cast<const bf16_t *>(a.w) + (static_cast<int64_t>(g) * kParts * a.n_out + (b / NB) * a.n_out + min(n0 + 16 * (b % NB) + r, a.n_out - 1)) * a.k;
    for (int m0 = blockIdx.z * 16 * MT; m0 < count; m0 += gridDim.z * 16 * MT) {
        const bf16_t *x[MT];
#pragma unroll
        for (int m = 0; m < MT; ++m)
            x[m] = static_cast<const bf16_t *>(a.x) + x_offset(a, g, group_row(a, g, min(m0 + 16 * m + r, count - 1)));
        f32x4_t acc[MT][kBlocks];
#pragma unroll
        for (int m = 0; m < MT; ++m)
#pragma unroll
            for (int b = 0; b < kBlocks; ++b) acc[m][b] = f32x4_t{0.f, 0.f, 0.f, 0.f};
        for (int s0 = s_begin; s0 < s_end; s0 += kAhead) {
            u32x4_t wf[kAhead][kBlocks], xf[kAhead][MT];
#pragma unroll
            for (int j = 0; j < kAhead; ++j) {
                const int e = (s0 + j) * 32 + 8 * q;
                const bool in = s0 + j < s_end && e < a.k;
#pragma unroll
                for (int b = 0; b < kBlocks; ++b) {
                    wf[j][b] = u32x4_t{0, 0, 0, 0};
                    if (in) wf[j][b] = *reinterpret_cast<const u32x4_t *>(w[b] + e);
                }
#pragma unroll
                for (int m = 0; m < MT; ++m) {
                    xf[j][m] = u32x4_t{0, 0, 0, 0};
                    if (in) xf[j][m] = *reinterpret_cast<const u32x4_t *>(x[m] + e);
                }
            }
#pragma unroll
            for (int j = 0; j < kAhead; ++j)
#pragma unroll
                for (int m = 0; m < MT; ++m)
#pragma unroll
                    for (int b = 0; b < kBlocks; ++b) acc[m][b] = mfma16(wf[j][b], xf[j][m], acc[m][b]);
        }
#pragma unroll
        for (int m = 0; m < MT; ++m)
#pragma unroll
            for (int b = 0; b < kBlocks; ++b) *reinterpret_cast<f32x4_t *>(&part[wave][16 * m + r][16 * b + 4 * q]) = acc[m][b];
        __syncthreads();
        for (int i = tid; i < MT * 16 * 16 * NB; i += 256) {
            const int m = i / (16 * NB), n = i % (16 * NB);
            if (m0 + m >= count || n0 + n >= a.n_out) continue;
            float v[kParts];
#pragma unroll
            for (int p = 0; p < kParts; ++p) {
                const int c = 16 * NB * p + n;
                v[p] = (part[0][m][c] + part[1][m][c]) + (part[2][m][c] + part[3][m][c]);
            }
            const int row = group_row(a, g, m0 + m);
            const float f = kGated ? input_weight(a, row) : 1.0f;
            static_cast<O *>(a.out)[out_offset(a, g, row) + n0 + n] =
                Elem<O>::from_f32(kGated ? gated_value<bf16_t>(a.gate, f * v[0], f * v[kParts - 1]) : result_of(a, v[0]));
        }
        __syncthreads();
    }
}

// ---- bf16, many rows per expert: tiles of BM rows x BN weight rows ----------------------------------
// Routed only.  A workgroup of four wavefronts (2 x 2) takes BM assignments of one expert and BN rows of its weights
// (gated: BN / 2 gates and the ups that belong to them, side by side in every wavefront).  Both operands travel
// global -> LDS without a register in between, in steps of 32 inner elements, and the wait before a barrier leaves
// later steps' loads in flight.  The LDS image is made of 1 KB blocks of 16 rows x 32 elements with the 16-byte pieces
// of a row permuted so that operand reads spread over the banks.  A CU gets some 18 bytes a clock out of the L2 for
// this, so the product per byte decides: 256 x 256 (one workgroup per CU, accumulators in accumulation registers, four
// buffers, a step's operands read while the step before it is multiplied) where there are enough rows and steps;
// otherwise 128 columns, three buffers and two or three workgroups per CU that cover for one another.
// Tiles are numbered expert by expert, eight row tiles abreast, and dealt out so that each XCD walks one stretch of that
// order: what runs together on it is about as many row tiles as weight tiles, which its L2 serves to all.
constexpr int kGroup = 8;

// Products of large tiles: the accumulators are asked for in accumulation registers, where the compiler would move
// them to and fro.  Nothing is known about the latency of these: products_done() before the results are read.
__device__ __forceinline__ void mfma16_in_place(const u32x4_t &x, const u32x4_t &y, f32x4_t &c) {
    asm("v_mfma_f32_16x16x32_bf16 %0, %1, %2, %0" : "+a"(c) : "v"(x), "v"(y));
}
template <int A, int B>
__device__ __forceinline__ void products_done(f32x4_t (&c)[A][B]) {
    auto tie = [&]() __attribute__((always_inline)) {        // neither products nor reads of their results cross it
#pragma unroll
        for (int i = 0; i < A; ++i)
#pragma unroll
            for (int j = 0; j < B; ++j) asm volatile("" : "+a"(c[i][j]));
    };
    tie();
    asm volatile("s_nop 15\n\ts_nop 15" ::: "memory");
    tie();
}

template <int BM, int BN, bool kGated>
__global__ __launch_bounds__(256, BN > 128 ? 1 : 2) void linear_tile_kernel(const LinearArgs a, const int32_t n_tiles) {
    constexpr bool kWide = BN > 128;
    constexpr int kTM = BM / 32, kTN = BN / 32;          // blocks of 16 per wavefront
    constexpr int kBlocksX = BM / 16, kBlocksW = BN / 16, kStage = (kBlocksX + kBlocksW) * 1024, kBuffers = kWide ? 4 : 3;
    constexpr int kLX = kBlocksX / 4, kLW = kBlocksW / 4, kLoads = kLX + kLW;   // blocks a wavefront loads per step
    __shared__ __attribute__((aligned(1024))) unsigned char smem[kBuffers * kStage];
    __shared__ int sh_row[BM];
    __shared__ float sh_weight[kGated ? BM : 1];
    const int tid = threadIdx.x, lane = tid & 63, r = lane & 15, g = lane >> 4;
    const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
    const int wm = wave & 1, wn = wave >> 1;
    // ---- which tile: row tiles of every expert, 64 experts at a time
    auto tiles_of = [&](int e) __attribute__((always_inline)) -> int { return e < a.groups ? (group_rows(a, e) + BM - 1) / BM : 0; };
    auto up_to = [&](int t) __attribute__((always_inline)) -> int {
#pragma unroll
        for (int d = 1; d < 64; d <<= 1) {
            const int o = __shfl_up(t, d, 64);
            if (lane >= d) t += o;
        }
        return t;
    };
    int own = tiles_of(lane), upto = up_to(own), total = __shfl(upto, 63, 64);
    for (int e0 = 64; e0 < a.groups; e0 += 64) total += __shfl(up_to(tiles_of(e0 + lane)), 63, 64);
    total = __builtin_amdgcn_readfirstlane(total) * n_tiles;
    const int stretch = (total + 7) / 8;
    const int in_stretch = blockIdx.x / 8;
    const int tile = blockIdx.x % 8 * stretch + in_stretch;
    if (in_stretch >= stretch || tile >= total) return;
    int m_tile = tile / n_tiles, expert = 0, m_tiles = 0;        // (first as if weight tiles were fastest, to find the expert)
    for (int e0 = 0;;) {
        const unsigned long long here = __ballot(m_tile < upto);
        if (here != 0) {
            const int first = __ffsll(here) - 1;
            expert = e0 + first;
            m_tiles = __shfl(own, first, 64);
            m_tile -= __shfl(upto, first, 64) - m_tiles;
            break;
        }
        m_tile -= __shfl(upto, 63, 64);
        e0 += 64;                                        // (m_tile < total: one of the experts has it)
        if (e0 >= a.groups) return;
        own = tiles_of(e0 + lane);
        upto = up_to(own);
    }
    expert = __builtin_amdgcn_readfirstlane(expert);
    m_tiles = __builtin_amdgcn_readfirstlane(m_tiles);
    // up to kGroup row tiles side by side, then the next weight tile
    const int at_expert = __builtin_amdgcn_readfirstlane(m_tile) * n_tiles + tile % n_tiles;
    const int group = at_expert / (kGroup * n_tiles), in_group = at_expert % (kGroup * n_tiles);
    const int abreast = min(kGroup, m_tiles - group * kGroup);
    const int n_tile = in_group / abreast;
    m_tile = group * kGroup + in_group % abreast;
    const int count = group_rows(a, expert), m0 = m_tile * BM;
    if (tid < BM) {                                      // (published by the barriers below)
        sh_row[tid] = group_row(a, expert, min(m0 + tid, count - 1));
        if constexpr (kGated) sh_weight[tid] = input_weight(a, sh_row[tid]);
    }

    // ---- what this wavefront loads: byte offsets of its lanes' pieces in the first step
    const int l16 = lane >> 2, piece = ((lane & 3) ^ ((0 - (l16 >> 2)) & 3)) * 8;
    uint32_t xoff[kLX], woff[kLW];
#pragma unroll
    for (int i = 0; i < kLX; ++i)
        xoff[i] = static_cast<uint32_t>(x_offset(a, expert, group_row(a, expert, min(m0 + 16 * (wave * kLX + i) + l16, count - 1))) + piece) * 2;
#pragma unroll
    for (int i = 0; i < kLW; ++i) {
        const int row = 16 * (wave * kLW + i) + l16;     // of the tile; gated: BN / 4 gates, their ups, twice
        int n;
        if (kGated) n = min(n_tile * (BN / 2) + row / (BN / 2) * (BN / 4) + row % (BN / 4), a.n_out - 1) + (row % (BN / 2) < BN / 4 ? 0 : a.n_out);
        else n = min(n_tile * BN + row, a.n_out - 1);
        woff[i] = static_cast<uint32_t>(n * static_cast<int64_t>(a.k) + piece) * 2;
    }
    const char *xb = static_cast<const char *>(a.x);
    const char *wb = static_cast<const char *>(a.w) + static_cast<int64_t>(expert) * (kGated ? 2 : 1) * a.n_out * a.k * 2;
    const lds_char_ptr lds = (lds_char_ptr)(&smem[0]);
    const uint32_t lds0 = __builtin_amdgcn_readfirstlane(static_cast<uint32_t>(reinterpret_cast<uintptr_t>(lds)));
    auto fetch = [&](int step, int buf) __attribute__((always_inline)) {
        const char *x = xb + 64 * static_cast<int64_t>(step), *w = wb + 64 * static_cast<int64_t>(step);
        const uint32_t at = lds0 + buf * kStage;
#pragma unroll
        for (int i = 0; i < kLX; ++i) load_to_lds_16(x, xoff[i], at + (wave * kLX + i) * 1024);
#pragma unroll
        for (int i = 0; i < kLW; ++i) load_to_lds_16(w, woff[i], at + (kBlocksX + wave * kLW + i) * 1024);
    };
    // the loads above are ordinary instructions to the compiler: this keeps them on their side of a barrier
    auto fence_loads = [&]() __attribute__((always_inline)) {
#pragma unroll
        for (int i = 0; i < kLX; ++i) asm volatile("" : "+v"(xoff[i]));
#pragma unroll
        for (int i = 0; i < kLW; ++i) asm volatile("" : "+v"(woff[i]));
    };
    // what step + kBuffers - 2 and later steps have asked for may still be on its way
    const int steps = a.k / 32;
    auto landed = [&](int step) __attribute__((always_inline)) {
        fence_loads();
        if (step + 1 < steps) asm volatile("s_waitcnt vmcnt(%0)" :: "i"(kLoads) : "memory");
        else asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
        __syncthreads();
        fence_loads();
    };

    f32x4_t acc[kTN][kTM];
#pragma unroll
    for (int n = 0; n < kTN; ++n)
#pragma unroll
        for (int m = 0; m < kTM; ++m) acc[n][m] = f32x4_t{0.f, 0.f, 0.f, 0.f};
    const lds_char_ptr frag = lds + 16 * (4 * r + (g ^ ((0 - (r >> 2)) & 3)));
    const lds_char_ptr xl = frag + wm * kTM * 1024, wl = frag + (kBlocksX + wn * kTN) * 1024;
    fetch(0, 0);
    if (steps > 1) fetch(1, 1);
    if constexpr (kWide) {
        u32x4_t wf[2][kTN], xf[2][kTM];                  // operands of even and odd steps
        auto read = [&](auto odd, int step) __attribute__((always_inline)) {
            constexpr int p = decltype(odd)::value;
            const int at = (step & 3) * kStage;
#pragma unroll
            for (int n = 0; n < kTN; ++n) wf[p][n] = *(lds_u32x4_ptr)(wl + at + n * 1024);
#pragma unroll
            for (int m = 0; m < kTM; ++m) xf[p][m] = *(lds_u32x4_ptr)(xl + at + m * 1024);
        };
        // the next step's data is there on every wavefront, a buffer nobody reads any more is filled, the next step's
        // operands are read, this step's are multiplied
        auto advance = [&](auto odd, int step) __attribute__((always_inline)) {
            constexpr int p = decltype(odd)::value;
            if (step + 1 < steps) {
                landed(step + 1);
                if (step + 3 < steps) fetch(step + 3, (step + 3) & 3);
                read(std::integral_constant<int, 1 - p>{}, step + 1);
            }
#pragma unroll
            for (int m = 0; m < kTM; ++m)
#pragma unroll
                for (int n = 0; n < kTN; ++n) mfma16_in_place(wf[p][n], xf[p][m], acc[n][m]);
        };
        constexpr std::integral_constant<int, 0> kEven{};
        constexpr std::integral_constant<int, 1> kOdd{};
        landed(0);
        if (steps > 2) fetch(2, 2);
        read(kEven, 0);
        int step = 0;
        for (; step + 1 < steps; step += 2) {
            advance(kEven, step);
            advance(kOdd, step + 1);
        }
        if (step < steps) advance(kEven, step);
        products_done(acc);
    } else {
        landed(0);
        int buf = 0;
        for (int step = 0; step < steps; ++step) {
            if (step + 2 < steps) fetch(step + 2, buf == 0 ? 2 : buf - 1);      // (the buffer of the step before this one)
            u32x4_t wf[kTN];
#pragma unroll
            for (int n = 0; n < kTN; ++n) wf[n] = *(lds_u32x4_ptr)(wl + buf * kStage + n * 1024);
#pragma unroll
            for (int m = 0; m < kTM; ++m) {
                const u32x4_t xf = *(lds_u32x4_ptr)(xl + buf * kStage + m * 1024);
#pragma unroll
                for (int n = 0; n < kTN; ++n) acc[n][m] = mfma16(wf[n], xf, acc[n][m]);
            }
            if (step + 1 < steps) landed(step + 1);
            buf = buf == 2 ? 0 : buf + 1;
        }
    }
    __syncthreads();                                     // everything has been read
    // ---- through LDS into whole pieces of rows (an accumulator holds four consecutive outputs of one row), the tile's
    // two halves of rows one after the other where all of it would not fit
    constexpr int kCols = kGated ? BN / 2 : BN, kOutPitch = kCols * 2 + 16, kPer = kCols / 8;
    constexpr int kRounds = BM * kOutPitch <= kBuffers * kStage ? 1 : 2;
    const int c = tid % kPer * 8, n0 = n_tile * kCols + c;
#pragma unroll
    for (int round = 0; round < kRounds; ++round) {
        if (kRounds == 1 || wm == round)
#pragma unroll
            for (int m = 0; m < kTM; ++m) {
                const float f = kGated ? sh_weight[16 * (wm * kTM + m) + r] : 1.0f;
#pragma unroll
                for (int n = 0; n < (kGated ? kTN / 2 : kTN); ++n) {
                    float y[4];
#pragma unroll
                    for (int j = 0; j < 4; ++j) y[j] = kGated ? gated_value<bf16_t>(a.gate, f * acc[n][m][j], f * acc[kGated ? n + kTN / 2 : n][m][j]) : acc[n][m][j];
                    *(__attribute__((address_space(3))) u32x2_t *)(lds + (16 * ((kRounds == 1 ? wm * kTM : 0) + m) + r) * kOutPitch + 2 * (kCols / 2 * wn + 16 * n + 4 * g)) =
                        u32x2_t{pack_bf16x2(y[0], y[1]), pack_bf16x2(y[2], y[3])};
                }
            }
        __syncthreads();
        const int base = round * (BM / 2), end = min(base + BM / kRounds, count - m0);
        if (n0 < a.n_out)
#pragma unroll 4
            for (int i = base + tid / kPer; i < end; i += 256 / kPer)            // (16-byte pieces)
                *reinterpret_cast<u32x4_t *>(static_cast<bf16_t *>(a.out) + static_cast<int64_t>(sh_row[i]) * a.o_stride + n0) = *(lds_u32x4_ptr)(lds + (i - base) * kOutPitch + 2 * c);
        if (kRounds > 1) __syncthreads();
    }
}

// Sizes the tiled form is built for: whole steps, whole 16-byte stores, 32-bit offsets.
static bool tiles_ok(const LinearArgs &a, bool gated, int32_t x_rows) {
    return a.k % 32 == 0 && a.n_out % 8 == 0 && aligned16(a.out) && static_cast<int64_t>(x_rows) * a.x_stride < (1LL << 30) &&
           static_cast<int64_t>(a.n_out) * (gated ? 2 : 1) * a.k < (1LL << 30);
}

template <int BM, int BN, bool kGated>
static int launch_tiles(const LinearArgs &a, hipStream_t s) {
    constexpr int kCols = kGated ? BN / 2 : BN;
    const int32_t n_tiles = (a.n_out + kCols - 1) / kCols;
    const int64_t most = (static_cast<int64_t>(a.rows) / BM + a.groups) * n_tiles;      // row tiles there can be, whatever the counts are
    const int64_t grid = (most + 7) / 8 * 8 + 8;
    if (grid > 0x7fffffffLL) return NVA_ERR_BAD_SHAPE;
    hipLaunchKernelGGL((linear_tile_kernel<BM, BN, kGated>), dim3(static_cast<uint32_t>(grid)), dim3(256), 0, s, a, n_tiles);
    return launch_status();
}

template <typename T, typename O, bool kGated>
static int launch_any_linear(const LinearArgs &a, int32_t most_rows, hipStream_t s) {
    const dim3 grid((a.n_out + 63) / 64, a.groups, std::min(std::max(1, (most_rows + 15) / 16), a.lists ? 64 : 65535));
    hipLaunchKernelGGL((linear_any_kernel<T, O, kGated>), grid, dim3(256), 0, s, a);
    return launch_status();
}

// rows_hint: rows a group is expected to have
template <int NB, bool kGated, typename O>
static int launch_skinny_nb(const LinearArgs &a, const LinearArgs &beside, int32_t rows_hint, int32_t most_rows, hipStream_t s) {
    const int mt = rows_hint <= 16 ? 1 : rows_hint <= 32 ? 2 : 4;
    const int passes = std::max(1, (most_rows + 16 * mt - 1) / (16 * mt));
    const dim3 grid((std::max(a.n_out, beside.n_out) + 16 * NB - 1) / (16 * NB), a.groups + beside.groups, a.lists && beside.groups == 0 ? 1 : std::min(passes, 65535)), block(256);
    if (mt == 1) hipLaunchKernelGGL((linear_skinny_kernel<1, NB, kGated, O>), grid, block, 0, s, a, beside);
    else if (mt == 2) hipLaunchKernelGGL((linear_skinny_kernel<2, NB, kGated, O>), grid, block, 0, s, a, beside);
    else hipLaunchKernelGGL((linear_skinny_kernel<4, NB, kGated, O>), grid, block, 0, s, a, beside);
    return launch_status();
}
template <bool kGated, typename O>
static int launch_skinny(const LinearArgs &a, int32_t rows_hint, int32_t most_rows, int32_t busy_groups, hipStream_t s,
                         const LinearArgs &beside = LinearArgs{}) {
    // two blocks of outputs per workgroup where that leaves enough workgroups for the machine
    if (static_cast<int64_t>(busy_groups) * ((a.n_out + 31) / 32) >= 512) return launch_skinny_nb<2, kGated, O>(a, beside, rows_hint, most_rows, s);
    return launch_skinny_nb<1, kGated, O>(a, beside, rows_hint, most_rows, s);
}

static bool linear_matrix_ok(const LinearArgs &a) {
    return a.k % 8 == 0 && a.x_stride % 8 == 0 && a.x_group % 8 == 0 && aligned16(a.x) && aligned16(a.w);
}

// ---- router ------------------------------------------------------------------------------------------

struct RouterArgs {
    const void *x;                   // [rows, width]
    int64_t x_stride;
    const void *w;                   // [experts + gates, width]
    const float *bias;               // [experts + gates] or null
    int32_t *choice;                 // [rows, top]
    float *weight;                   // [rows, top + gates]: the choices' weights, the gates' sigmoids
    int32_t *lists, *counts;         // [experts, list_stride], [experts] (zero on entry)
    int64_t list_stride;
    int32_t rows, width, experts, gates, top;
    int32_t sigmoid;                 // weights: the chosen logits' sigmoids
    float scale;
};

// 16 TG rows per workgroup of NW wavefronts; KS = NW / TG wavefronts share a group's inner dimension.
constexpr float kWeightGuard = 1e-20f;

template <typename T, int TG, int NW, bool kMatrix>
__global__ __launch_bounds__(64 * NW) void router_kernel(RouterArgs a) {
    constexpr int KS = NW / TG, kRows = 16 * TG, kThreads = 64 * NW;
    extern __shared__ __attribute__((aligned(16))) unsigned char router_smem[];
    const int outs = a.experts + a.gates;
    float *logits = reinterpret_cast<float *>(router_smem);                    // [kRows][outs]
    float *partial = logits + kRows * outs;                                    // [KS][kRows][64 + 4] (matrix form)
    int *have = reinterpret_cast<int *>(partial + (kMatrix ? KS * kRows * 68 : 0)); // [experts]: this workgroup's assignments
    int *base = have + a.experts;                                              // [experts]
    int *mine = base + a.experts;                                              // [kRows * top]: expert, place among this workgroup's
    const int tid = threadIdx.x, lane = tid & 63, r = lane & 15, q = lane >> 4;
    const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
    const int row0 = blockIdx.x * kRows;
    const int rows = min(kRows, a.rows - row0);
    for (int e = tid; e < a.experts; e += kThreads) have[e] = 0;
    if constexpr (kMatrix) {
        const int tg = wave / KS, part = wave % KS;
        const int steps = (a.width + 31) / 32, per = (steps + KS - 1) / KS;
        const int s_begin = part * per, s_end = min(steps, s_begin + per);
        const bf16_t *x = static_cast<const bf16_t *>(a.x) + static_cast<int64_t>(row0 + min(16 * tg + r, rows - 1)) * a.x_stride;
        for (int e0 = 0; e0 < outs; e0 += 64) {
            const int blocks = min(4, (outs - e0 + 15) / 16);
            f32x4_t acc[4];
            const bf16_t *w[4];
#pragma unroll
            for (int b = 0; b < 4; ++b) {
                acc[b] = f32x4_t{0.f, 0.f, 0.f, 0.f};
                w[b] = static_cast<const bf16_t *>(a.w) + static_cast<int64_t>(min(e0 + 16 * b + r, outs - 1)) * a.width;
            }
            for (int s = s_begin; s < s_end; ++s) {
                const int e = s * 32 + 8 * q;
                const bool in = e < a.width;
                u32x4_t xf = {0, 0, 0, 0};
                if (in) xf = *reinterpret_cast<const u32x4_t *>(x + e);
#pragma unroll
                for (int b = 0; b < 4; ++b) {
                    u32x4_t wf = {0, 0, 0, 0};
                    if (in && b < blocks) wf = *reinterpret_cast<const u32x4_t *>(w[b] + e);
                    acc[b] = mfma16(wf, xf, acc[b]);
                }
            }
#pragma unroll
            for (int b = 0; b < 4; ++b) *reinterpret_cast<f32x4_t *>(partial + (part * kRows + 16 * tg + r) * 68 + 16 * b + 4 * q) = acc[b];
            __syncthreads();
            for (int i = tid; i < kRows * 64; i += kThreads) {
                const int row = i >> 6, e = i & 63;
                if (e0 + e >= outs) continue;
                float z = a.bias != nullptr ? a.bias[e0 + e] : 0.f;
#pragma unroll
                for (int p = 0; p < KS; ++p) z += partial[(p * kRows + row) * 68 + e];
                logits[row * outs + e0 + e] = z;
            }
            __syncthreads();
        }
    } else {
        for (int i = tid; i < rows * outs; i += kThreads) {
            const int row = i / outs, e = i % outs;
            const T *x = static_cast<const T *>(a.x) + static_cast<int64_t>(row0 + row) * a.x_stride;
            const T *w = static_cast<const T *>(a.w) + static_cast<int64_t>(e) * a.width;
            float z = a.bias != nullptr ? a.bias[e] : 0.f;
            for (int k = 0; k < a.width; ++k) z = fmaf(Elem<T>::to_f32(x[k]), Elem<T>::to_f32(w[k]), z);
            logits[i] = z;
        }
        __syncthreads();
    }
    // one wavefront per row: softmax over the experts (or their sigmoids; both rise with the logit), then the best one `top`
    // times (ties: the lower index)
    for (int row = wave; row < rows; row += NW) {
        float *z = logits + row * outs;
        float mine_z = -INFINITY, mx = -INFINITY;            // (up to 64 experts: one per lane)
        const bool narrow = a.experts <= 64;
        if (narrow) {
            if (lane < a.experts) mine_z = z[lane];
            mx = mine_z;
        } else {
            for (int e = lane; e < a.experts; e += 64) mx = fmaxf(mx, z[e]);
        }
        mx = wave_max(mx);
        float sum = 0.f;
        if (narrow) sum = exp_of<T>(mine_z - mx);
        else for (int e = lane; e < a.experts; e += 64) sum += exp_of<T>(z[e] - mx);
        const float inv = 1.0f / wave_sum(sum);
        float chosen = 0.f, my_s = 0.f;                    // lane k keeps choice k (of every 64)
        int my_who = 0;
        for (int k = 0; k < a.top; ++k) {
            float best = mine_z;
            int who = lane;
            if (!narrow) {
                best = -INFINITY;
                for (int e = lane; e < a.experts; e += 64)
                    if (z[e] > best) { best = z[e]; who = e; }
            }
            const float best_now = wave_max(best);
            const unsigned long long at = __ballot(best == best_now);
            int win;
            if (narrow) win = at != 0 ? __ffsll(at) - 1 : 0;
            else win = 1023 - static_cast<int>(wave_max(best == best_now ? static_cast<float>(1023 - who) : 0.f));
            if (win >= a.experts) win = 0;                   // (only where logits are not numbers)
            const float s = a.sigmoid ? sigmoid_of<T>(best_now) : exp_of<T>(best_now - mx) * inv;
            chosen += s;
            if (lane == k % 64) {
                my_s = s;
                my_who = win;
            }
            if (narrow) { if (lane == win) mine_z = -INFINITY; }
            else {
                if (lane == 0) z[win] = -INFINITY;
                __builtin_amdgcn_fence(__ATOMIC_ACQ_REL, "wavefront");
            }
            if (k % 64 == 63 || k == a.top - 1) {            // hand over up to 64 choices at once
                const int kk = k / 64 * 64 + lane;
                if (kk <= k) {
                    mine[2 * (row * a.top + kk)] = my_who;
                    mine[2 * (row * a.top + kk) + 1] = __float_as_int(my_s);
                }
            }
        }
        __builtin_amdgcn_fence(__ATOMIC_ACQ_REL, "wavefront");
        const float f = a.sigmoid ? a.scale : a.scale / (chosen + kWeightGuard);
        const int64_t at = static_cast<int64_t>(row0 + row) * a.top;
        float *out = a.weight + static_cast<int64_t>(row0 + row) * (a.top + a.gates);
        for (int j = lane; j < a.gates; j += 64) out[a.top + j] = sigmoid_of<T>(z[a.experts + j]);
        for (int k = lane; k < a.top; k += 64) {
            const int who = mine[2 * (row * a.top + k)];
            a.choice[at + k] = who;
            out[k] = __int_as_float(mine[2 * (row * a.top + k) + 1]) * f;
            mine[2 * (row * a.top + k) + 1] = atomicAdd(&have[who], 1);
        }
    }
    __syncthreads();
    const bool alone = gridDim.x == 1;                       // nobody else adds to the counters
    for (int e = tid; e < a.experts; e += kThreads) {
        base[e] = 0;
        if (alone) a.counts[e] = have[e];
        else if (have[e] > 0) base[e] = atomicAdd(&a.counts[e], have[e]);
    }
    __syncthreads();
    for (int i = tid; i < rows * a.top; i += kThreads) {
        const int e = mine[2 * i], place = base[e] + mine[2 * i + 1];
        if (place < a.list_stride) a.lists[e * a.list_stride + place] = row0 * a.top + i;
    }
}

static size_t router_lds(int32_t experts, int32_t gates, int32_t top, int tg, int nw, bool matrix) {
    const size_t rows = 16 * static_cast<size_t>(tg);
    return 4 * (rows * (experts + gates) + (matrix ? nw / tg * rows * 68 : 0) + 2 * static_cast<size_t>(experts) + 2 * rows * top);
}

template <typename T, int TG, int NW, bool kMatrix>
static int launch_router_tg(const RouterArgs &a, hipStream_t s) {
    const size_t lds = router_lds(a.experts, a.gates, a.top, TG, NW, kMatrix);
    if (lds > 64 * 1024 &&
        hipFuncSetAttribute(reinterpret_cast<const void *>(&router_kernel<T, TG, NW, kMatrix>), hipFuncAttributeMaxDynamicSharedMemorySize, static_cast<int>(lds)) != hipSuccess)
        return NVA_ERR_LAUNCH_FAILED;
    hipLaunchKernelGGL((router_kernel<T, TG, NW, kMatrix>), dim3((a.rows + 16 * TG - 1) / (16 * TG)), dim3(64 * NW), lds, s, a);
    return launch_status();
}

}  // namespace nva

extern "C" int nva_grouped_linear(const void *x, int64_t x_row_stride, int64_t x_group_stride, const void *weight, void *out,
                                  int64_t out_row_stride, int64_t out_group_stride, int32_t rows, int32_t groups, int32_t n_out,
                                  int32_t k_in, int32_t squared_relu, int32_t dtype, int32_t out_dtype, void *stream) {
    using namespace nva;
    if (rows < 0 || groups < 0 || n_out <= 0 || k_in <= 0) return NVA_ERR_BAD_SHAPE;
    if (!known_dtype(dtype) || !known_dtype(out_dtype) || (dtype == NVA_DTYPE_F32 && out_dtype != NVA_DTYPE_F32)) return NVA_ERR_UNSUPPORTED_GEOMETRY;
    if (rows == 0 || groups == 0) return NVA_OK;
    if (!x || !weight || !out) return NVA_ERR_NULL_POINTER;
    if (groups > 65535) return NVA_ERR_BAD_SHAPE;
    if (x_row_stride < k_in || out_row_stride < n_out || (groups > 1 && (x_group_stride < 0 || out_group_stride < n_out))) return NVA_ERR_BAD_STRIDE;
    LinearArgs a{};
    a.x = x; a.x_stride = x_row_stride; a.x_group = groups > 1 ? x_group_stride : 0; a.w = weight; a.out = out; a.o_stride = out_row_stride;
    a.o_group = groups > 1 ? out_group_stride : 0; a.rows = rows; a.groups = groups; a.n_out = n_out; a.k = k_in; a.x_div = 1; a.squared_relu = squared_relu;
    hipStream_t s = static_cast<hipStream_t>(stream);
    if (dtype == NVA_DTYPE_F32) return launch_any_linear<float, float, false>(a, rows, s);
    if (!linear_matrix_ok(a))
        return out_dtype == NVA_DTYPE_F32 ? launch_any_linear<bf16_t, float, false>(a, rows, s) : launch_any_linear<bf16_t, bf16_t, false>(a, rows, s);
    return out_dtype == NVA_DTYPE_F32 ? launch_skinny<false, float>(a, rows, rows, groups, s) : launch_skinny<false, bf16_t>(a, rows, rows, groups, s);
}

namespace nva {
static int routed_args(LinearArgs &a, const void *x, int64_t x_row_stride, const void *weight, void *out, const int32_t *lists,
                       const int32_t *counts, int64_t list_stride, int32_t rows, int32_t terms, int32_t experts, int32_t n_out,
                       int32_t k_in, int32_t x_per_row, float gate_limit, float gate_slope, float gate_shift, const float *in_weight,
                       int64_t in_weight_row_stride, int32_t dtype) {
    if (rows < 0 || terms <= 0 || experts <= 0 || n_out <= 0 || k_in <= 0 || list_stride < rows || terms > experts) return NVA_ERR_BAD_SHAPE;
    if (!known_dtype(dtype)) return NVA_ERR_UNSUPPORTED_GEOMETRY;
    if (rows == 0) return NVA_OK;
    if (!x || !weight || !out || !lists || !counts) return NVA_ERR_NULL_POINTER;
    if (experts > 65535 || static_cast<int64_t>(rows) * terms > 0x7fffffffLL) return NVA_ERR_BAD_SHAPE;
    if (x_row_stride < k_in || (in_weight && in_weight_row_stride < terms)) return NVA_ERR_BAD_STRIDE;
    a.in_weight = in_weight; a.in_stride = in_weight_row_stride; a.terms = terms;
    a.x = x; a.x_stride = x_row_stride; a.w = weight; a.out = out; a.o_stride = n_out; a.lists = lists; a.counts = counts;
    a.list_stride = list_stride; a.rows = rows * terms; a.groups = experts; a.n_out = n_out; a.k = k_in; a.x_div = x_per_row ? terms : 1;
    a.gate = GateForm{gate_limit, gate_slope, gate_shift};
    return NVA_OK;
}
static int32_t rows_hint_of(int32_t rows, int32_t terms, int32_t experts) {
    return static_cast<int32_t>((static_cast<int64_t>(rows) * terms * 3 / 2 + experts - 1) / experts);
}
static int32_t busy_experts(int32_t rows, int32_t terms, int32_t experts) {
    return static_cast<int32_t>(std::min(static_cast<int64_t>(experts), static_cast<int64_t>(rows) * terms));
}
}  // namespace nva

extern "C" int nva_routed_linear(const void *x, int64_t x_row_stride, const void *weight, void *out, const int32_t *lists,
                                 const int32_t *counts, int64_t list_stride, int32_t rows, int32_t terms, int32_t experts,
                                 int32_t n_out, int32_t k_in, int32_t x_per_row, int32_t gated, float gate_limit, float gate_slope, float gate_shift,
                                 const float *in_weight, int64_t in_weight_row_stride, int32_t dtype, void *stream) {
    using namespace nva;
    if (in_weight && !gated) return NVA_ERR_UNSUPPORTED_GEOMETRY;
    LinearArgs a{};
    const int rc = routed_args(a, x, x_row_stride, weight, out, lists, counts, list_stride, rows, terms, experts, n_out, k_in, x_per_row,
                               gate_limit, gate_slope, gate_shift, in_weight, in_weight_row_stride, dtype);
    if (rc != NVA_OK || rows == 0) return rc;
    hipStream_t s = static_cast<hipStream_t>(stream);
    if (dtype == NVA_DTYPE_F32) return gated ? launch_any_linear<float, float, true>(a, rows, s) : launch_any_linear<float, float, false>(a, rows, s);
    if (!linear_matrix_ok(a)) return gated ? launch_any_linear<bf16_t, bf16_t, true>(a, rows, s) : launch_any_linear<bf16_t, bf16_t, false>(a, rows, s);
    const int32_t average = static_cast<int32_t>(static_cast<int64_t>(rows) * terms / experts);
    if (average >= 48 && tiles_ok(a, gated, x_per_row ? rows : rows * terms)) {
        if (average >= 512 && k_in >= 1536) return gated ? launch_tiles<256, 256, true>(a, s) : launch_tiles<256, 256, false>(a, s);
        if (average >= 512) return gated ? launch_tiles<256, 128, true>(a, s) : launch_tiles<256, 128, false>(a, s);
        return gated ? launch_tiles<128, 128, true>(a, s) : launch_tiles<128, 128, false>(a, s);
    }
    const int32_t hint = rows_hint_of(rows, terms, experts), busy = busy_experts(rows, terms, experts);
    return gated ? launch_skinny<true, bf16_t>(a, hint, rows, busy, s) : launch_skinny<false, bf16_t>(a, hint, rows, busy, s);
}

extern "C" int nva_routed_shared_linear(const void *x, int64_t x_row_stride, const void *weight, void *out, const int32_t *lists,
                                        const int32_t *counts, int64_t list_stride, int32_t rows, int32_t terms, int32_t experts,
                                        int32_t n_out, int32_t k_in, int32_t x_per_row, int32_t gated, float gate_limit, float gate_slope,
                                        float gate_shift, const void *shared_x, int64_t shared_x_row_stride, const void *shared_weight,
                                        void *shared_out, int32_t shared_n_out, int32_t shared_k_in, float shared_gate_limit, void *stream) {
    using namespace nva;
    LinearArgs a{}, b{};
    const int rc = routed_args(a, x, x_row_stride, weight, out, lists, counts, list_stride, rows, terms, experts, n_out, k_in, x_per_row,
                               gate_limit, gate_slope, gate_shift, nullptr, 0, NVA_DTYPE_BF16);
    if (rc != NVA_OK) return rc;
    if (shared_n_out <= 0 || shared_k_in <= 0) return NVA_ERR_BAD_SHAPE;
    if (rows == 0) return NVA_OK;
    if (!shared_x || !shared_weight || !shared_out) return NVA_ERR_NULL_POINTER;
    if (shared_x_row_stride < shared_k_in) return NVA_ERR_BAD_STRIDE;
    b.x = shared_x; b.x_stride = shared_x_row_stride; b.w = shared_weight; b.out = shared_out; b.o_stride = shared_n_out; b.rows = rows; b.groups = 1;
    b.n_out = shared_n_out; b.k = shared_k_in; b.x_div = 1; b.gate = GateForm{shared_gate_limit, gate_slope, gate_shift};
    if (!linear_matrix_ok(a) || !linear_matrix_ok(b)) return NVA_ERR_UNSUPPORTED_GEOMETRY;
    hipStream_t s = static_cast<hipStream_t>(stream);
    const int32_t hint = rows_hint_of(rows, terms, experts), busy = busy_experts(rows, terms, experts);
    return gated ? launch_skinny<true, bf16_t>(a, hint, rows, busy, s, b) : launch_skinny<false, bf16_t>(a, hint, rows, busy, s, b);
}

extern "C" int nva_router(const void *x, int64_t x_row_stride, const void *weight, const float *bias, int32_t *choice,
                          float *choice_weight, int32_t *lists, int32_t *counts, int64_t list_stride, int32_t rows, int32_t width,
                          int32_t experts, int32_t gates, int32_t top, int32_t score, float scale, int32_t dtype, void *stream) {
    using namespace nva;
    if (score != NVA_SCORE_SOFTMAX && score != NVA_SCORE_SIGMOID) return NVA_ERR_UNSUPPORTED_GEOMETRY;
    if (rows < 0 || width <= 0 || experts <= 0 || gates < 0 || top <= 0 || top > experts || list_stride < rows) return NVA_ERR_BAD_SHAPE;
    if (!known_dtype(dtype) || experts > 1024 || gates > 64 || top > 128) return NVA_ERR_UNSUPPORTED_GEOMETRY;
    if (rows == 0) return NVA_OK;
    if (!x || !weight || !choice || !choice_weight || !lists || !counts) return NVA_ERR_NULL_POINTER;
    if (x_row_stride < width) return NVA_ERR_BAD_STRIDE;
    if (static_cast<int64_t>(rows) * top > 0x7fffffffLL) return NVA_ERR_BAD_SHAPE;
    RouterArgs a{};
    a.x = x; a.x_stride = x_row_stride; a.w = weight; a.bias = bias; a.choice = choice; a.weight = choice_weight; a.lists = lists; a.counts = counts;
    a.list_stride = list_stride; a.rows = rows; a.width = width; a.experts = experts; a.gates = gates; a.top = top; a.sigmoid = score == NVA_SCORE_SIGMOID; a.scale = scale;
    hipStream_t s = static_cast<hipStream_t>(stream);
    const bool many = rows >= 4096 && experts <= 128 && top <= 32;       // more rows per workgroup: fewer additions to the counters
    if (dtype == NVA_DTYPE_F32) return launch_router_tg<float, 1, 8, false>(a, s);
    if (width % 8 != 0 || x_row_stride % 8 != 0 || !aligned16(x) || !aligned16(weight)) return launch_router_tg<bf16_t, 1, 8, false>(a, s);
    if (many) return launch_router_tg<bf16_t, 4, 8, true>(a, s);
    return rows <= 1024 && experts <= 256 ? launch_router_tg<bf16_t, 1, 16, true>(a, s) : launch_router_tg<bf16_t, 1, 8, true>(a, s);
}
