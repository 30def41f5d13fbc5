// Fused steps between the matrix products of layered models with an fp32 residual stream:
//   embed_norm        residual = embed[id] * scale; out = layer_norm(residual)
//   post_add_norm     residual += layer_norm(y); out = layer_norm'(residual)     (the norm after a
//                     sublayer, the residual add and the norm before the next one in one kernel)
//   conv_rope_store   short causal convolution of q, k and v, rotary embedding of q and k, cache write
//   conv_state_update the last taps - 1 projected rows of every portion, kept for the next one
// Tensors are bf16 or fp32 (one template argument); every sum, norm and angle is fp32.
#include "nva_elem.h"

#include <math.h>

namespace nva {

// ---- layer norms around the residual stream ----------------------------------------------------

struct NormArgs {
    const int64_t *ids;          // embed: token ids [rows]
    const void *x;               // embed: table [vocab, width]; otherwise y [*, width]
    int64_t x_stride;
    float *residual;             // fp32 [*, width] dense
    const void *w_post, *b_post; // norm of y (not used by embed)
    const void *w_next, *b_next; // norm of the new residual
    void *out;                   // [rows, width] dense
    const int32_t *rows_of;      // optional: output row r is computed from row rows_of[r], residual left alone
    int32_t rows, src_rows, width, vocab;
    float scale, eps;
};

__device__ __forceinline__ int64_t norm_source_row(const NormArgs &a, int row, bool embed) {
    if (embed || a.rows_of == nullptr) return row;
    return min(max(a.rows_of[row], 0), a.src_rows - 1);      // device data the host could not check
}

// One wavefront per row, the row in registers; NC pieces of 512 elements (width % 8 == 0, width <= 4096).
template <typename T, int NC, bool kEmbed>
__global__ __launch_bounds__(256) void norm_rows_kernel(NormArgs a) {
    const int lane = threadIdx.x & 63;
    const int row = blockIdx.x * 4 + (threadIdx.x >> 6);
    if (row >= a.rows) return;
    const int64_t src = norm_source_row(a, row, kEmbed);
    int64_t xrow = src;
    if (kEmbed) xrow = min(max(a.ids[row], static_cast<int64_t>(0)), static_cast<int64_t>(a.vocab) - 1);
    const T *xp = static_cast<const T *>(a.x) + xrow * a.x_stride;
    float *rp = a.residual + src * a.width;
    float v[NC][8], r[NC][8];
#pragma unroll
    for (int c = 0; c < NC; ++c) {
        const int e = min(c * 512 + lane * 8, a.width - 8);  // lanes past the row re-read its end
        load_f32<T, 8>(xp + e, v[c]);
        if (!kEmbed) load_f32<float, 8>(rp + e, r[c]);
    }
    const float inv_n = 1.0f / static_cast<float>(a.width);
    if (kEmbed) {
#pragma unroll
        for (int c = 0; c < NC; ++c)
#pragma unroll
            for (int i = 0; i < 8; ++i) r[c][i] = v[c][i] * a.scale;
    } else {
        float sum = 0.f;
#pragma unroll
        for (int c = 0; c < NC; ++c)
            if (c * 512 + lane * 8 < a.width)
#pragma unroll
                for (int i = 0; i < 8; ++i) sum += v[c][i];
        const float mean = wave_sum(sum) * inv_n;
        float sq = 0.f;
#pragma unroll
        for (int c = 0; c < NC; ++c)
            if (c * 512 + lane * 8 < a.width)
#pragma unroll
                for (int i = 0; i < 8; ++i) { const float d = v[c][i] - mean; sq = fmaf(d, d, sq); }
        const float rstd = rsqrtf(wave_sum(sq) * inv_n + a.eps);
#pragma unroll
        for (int c = 0; c < NC; ++c) {
            const int e = min(c * 512 + lane * 8, a.width - 8);
            float w[8], b[8];
            load_f32<T, 8>(static_cast<const T *>(a.w_post) + e, w);
            load_f32<T, 8>(static_cast<const T *>(a.b_post) + e, b);
#pragma unroll
            for (int i = 0; i < 8; ++i) r[c][i] += fmaf((v[c][i] - mean) * rstd, w[i], b[i]);
        }
    }
    float sum = 0.f;
#pragma unroll
    for (int c = 0; c < NC; ++c) {
        const int e = c * 512 + lane * 8;
        if (e < a.width) {
            if (kEmbed || a.rows_of == nullptr) store_f32<float, 8>(rp + e, r[c]);
#pragma unroll
            for (int i = 0; i < 8; ++i) sum += r[c][i];
        }
    }
    const float mean = wave_sum(sum) * inv_n;
    float sq = 0.f;
#pragma unroll
    for (int c = 0; c < NC; ++c)
        if (c * 512 + lane * 8 < a.width)
#pragma unroll
            for (int i = 0; i < 8; ++i) { const float d = r[c][i] - mean; sq = fmaf(d, d, sq); }
    const float rstd = rsqrtf(wave_sum(sq) * inv_n + a.eps);
    T *op = static_cast<T *>(a.out) + static_cast<int64_t>(row) * a.width;
#pragma unroll
    for (int c = 0; c < NC; ++c) {
        const int e = c * 512 + lane * 8;
        if (e < a.width) {
            float w[8], b[8], y[8];
            load_f32<T, 8>(static_cast<const T *>(a.w_next) + e, w);
            load_f32<T, 8>(static_cast<const T *>(a.b_next) + e, b);
#pragma unroll
            for (int i = 0; i < 8; ++i) y[i] = fmaf((r[c][i] - mean) * rstd, w[i], b[i]);
            store_f32<T, 8>(op + e, y);
        }
    }
}

__device__ __forceinline__ float block_sum_256(float v, float *sh) {
    v = wave_sum(v);
    __syncthreads();
    if ((threadIdx.x & 63) == 0) sh[threadIdx.x >> 6] = v;
    __syncthreads();
    return (sh[0] + sh[1]) + (sh[2] + sh[3]);
}

// Any width: one workgroup per row, the row is read again for every pass (it sits in L2); the values
// of the new residual are recomputed rather than kept.
template <typename T, bool kEmbed>
__global__ __launch_bounds__(256) void norm_rows_any_kernel(NormArgs a) {
    __shared__ float sh[4];
    const int row = blockIdx.x;
    const int64_t src = norm_source_row(a, row, kEmbed);
    int64_t xrow = src;
    if (kEmbed) xrow = min(max(a.ids[row], static_cast<int64_t>(0)), static_cast<int64_t>(a.vocab) - 1);
    const T *xp = static_cast<const T *>(a.x) + xrow * a.x_stride;
    float *rp = a.residual + src * a.width;
    const T *wp = static_cast<const T *>(a.w_post), *bp = static_cast<const T *>(a.b_post);
    const T *wn = static_cast<const T *>(a.w_next), *bn = static_cast<const T *>(a.b_next);
    const float inv_n = 1.0f / static_cast<float>(a.width);
    float mean1 = 0.f, rstd1 = 0.f;
    if (!kEmbed) {
        float s = 0.f;
        for (int e = threadIdx.x; e < a.width; e += 256) s += Elem<T>::to_f32(xp[e]);
        mean1 = block_sum_256(s, sh) * inv_n;
        s = 0.f;
        for (int e = threadIdx.x; e < a.width; e += 256) { const float d = Elem<T>::to_f32(xp[e]) - mean1; s = fmaf(d, d, s); }
        rstd1 = rsqrtf(block_sum_256(s, sh) * inv_n + a.eps);
    }
    auto value = [&](int e) -> float {
        const float x = Elem<T>::to_f32(xp[e]);
        if (kEmbed) return x * a.scale;
        return rp[e] + fmaf((x - mean1) * rstd1, Elem<T>::to_f32(wp[e]), Elem<T>::to_f32(bp[e]));
    };
    float s = 0.f;
    for (int e = threadIdx.x; e < a.width; e += 256) s += value(e);
    const float mean = block_sum_256(s, sh) * inv_n;
    s = 0.f;
    for (int e = threadIdx.x; e < a.width; e += 256) { const float d = value(e) - mean; s = fmaf(d, d, s); }
    const float rstd = rsqrtf(block_sum_256(s, sh) * inv_n + a.eps);
    T *op = static_cast<T *>(a.out) + static_cast<int64_t>(row) * a.width;
    for (int e = threadIdx.x; e < a.width; e += 256) {
        const float r = value(e);                            // (before this thread overwrites rp[e])
        if (kEmbed || a.rows_of == nullptr) rp[e] = r;
        op[e] = Elem<T>::from_f32(fmaf((r - mean) * rstd, Elem<T>::to_f32(wn[e]), Elem<T>::to_f32(bn[e])));
    }
}

template <typename T, bool kEmbed>
static void launch_norm(const NormArgs &a, bool vector, hipStream_t s) {
    if (!vector) {
        hipLaunchKernelGGL((norm_rows_any_kernel<T, kEmbed>), dim3(a.rows), dim3(256), 0, s, a);
        return;
    }
    const dim3 grid((a.rows + 3) / 4), block(256);
    switch ((a.width + 511) / 512) {
        case 1: hipLaunchKernelGGL((norm_rows_kernel<T, 1, kEmbed>), grid, block, 0, s, a); break;
        case 2: hipLaunchKernelGGL((norm_rows_kernel<T, 2, kEmbed>), grid, block, 0, s, a); break;
        case 3: case 4: hipLaunchKernelGGL((norm_rows_kernel<T, 4, kEmbed>), grid, block, 0, s, a); break;
        default: hipLaunchKernelGGL((norm_rows_kernel<T, 8, kEmbed>), grid, block, 0, s, a); break;
    }
}

static bool norm_vector_ok(const NormArgs &a) {
    return a.width % 8 == 0 && a.width <= 4096 && a.x_stride % 8 == 0 && aligned16(a.x) && aligned16(a.residual) &&
           aligned16(a.w_post) && aligned16(a.b_post) && aligned16(a.w_next) && aligned16(a.b_next) && aligned16(a.out);
}

// ---- short convolution + rotary embedding + cache write ---------------------------------------------

struct ConvRopeArgs {
    const void *qkv;                // [n, (H + G) * dim + G * vdim], row stride in elements
    int64_t stride;
    const void *weight;             // [taps, channels]: tap taps - 1 meets the row itself
    void *state;                    // [state_slots, taps - 1, channels]: oldest row first (null when taps == 1)
    const int32_t *slots_of_seq;    // state slot of every sequence
    const int32_t *cu;              // portions: [n_seqs + 1] row bounds
    const int32_t *klen;            // tokens of every sequence once its rows are in (decode: 0 = padded row)
    const int32_t *token_seq;       // portions: sequence of every row
    const float *rope;              // [max_position, rot_dims]: cos | sin
    void *q_out;                    // [n, H * dim]
    void *k_cache, *v_cache;        // flat [num_slots, G * dim], [num_slots, G * vdim]
    const int32_t *slot_mapping;    // [n]
    int64_t num_slots;
    int32_t n, n_seqs, heads, kv_heads, dim, vdim, half, taps, max_position, state_slots;
};

// A thread owns one group of V channels (two groups, i and i + half, where the rotation pairs them) and
// walks kTokens consecutive rows with the taps - 1 rows before it in registers and the next row on its way.
// kTaps >= taps: missing old taps have weight zero and are not read.  kDecode: every row is a sequence of
// its own, and the thread also shifts its channels of the carried rows.
template <typename T, int kTaps, int V, int kTokens, bool kDecode>
__global__ __launch_bounds__(256) void conv_rope_store_kernel(ConvRopeArgs a) {
    constexpr int kHist = kTaps - 1;
    const int pairs = a.half / V, rest = (a.dim - 2 * a.half) / V, per_head = pairs + rest;
    const int qk_units = (a.heads + a.kv_heads) * per_head;
    const int v_per_head = a.vdim / V;
    const int units = qk_units + a.kv_heads * v_per_head;
    const int64_t idx = static_cast<int64_t>(blockIdx.x) * 256 + threadIdx.x;
    const int64_t t0 = idx / units * kTokens;
    if (t0 >= a.n) return;
    const int u = static_cast<int>(idx % units);
    int head, off, ri = 0;
    bool pair = false;
    const bool is_v = u >= qk_units;
    if (is_v) {
        head = (u - qk_units) / v_per_head;
        off = (u - qk_units) % v_per_head * V;
    } else {
        head = u / per_head;
        const int w = u % per_head;
        pair = w < pairs;
        ri = w * V;
        off = pair ? ri : 2 * a.half + (w - pairs) * V;
    }
    const int64_t channels = static_cast<int64_t>(a.heads + a.kv_heads) * a.dim + static_cast<int64_t>(a.kv_heads) * a.vdim;
    const int64_t c0 = is_v ? static_cast<int64_t>(a.heads + a.kv_heads) * a.dim + static_cast<int64_t>(head) * a.vdim + off
                            : static_cast<int64_t>(head) * a.dim + off;
    const int64_t c1 = pair ? c0 + a.half : c0;
    const T *qkv = static_cast<const T *>(a.qkv);
    T *state = static_cast<T *>(a.state);
    const int t_end = static_cast<int>(min(static_cast<int64_t>(a.n), t0 + kTokens));

    // the sequence of the first row: its rows [first, row_end), its tokens before them
    int seq, first, row_end, start, slot_s;
    auto enter = [&](int s) __attribute__((always_inline)) {
        seq = s;
        if (kDecode) {
            first = seq;
            row_end = seq + 1;
            start = a.klen[seq] - 1;
        } else {
            first = a.cu[seq];
            row_end = a.cu[seq + 1];
            start = a.klen[seq] - (row_end - first);
        }
        slot_s = a.taps > 1 ? a.slots_of_seq[seq] : -1;
    };
    enter(kDecode ? static_cast<int>(t0) : min(max(a.token_seq[t0], 0), a.n_seqs - 1));
    if (kDecode && start < 0) {                           // padded row of a batch bucket
        float zero[V];
#pragma unroll
        for (int i = 0; i < V; ++i) zero[i] = 0.f;
        if (!is_v && head < a.heads) {
            T *q = static_cast<T *>(a.q_out) + t0 * a.heads * a.dim + static_cast<int64_t>(head) * a.dim + off;
            store_f32<T, V>(q, zero);
            if (pair) store_f32<T, V>(q + a.half, zero);
        }
        return;
    }

    float w0[kTaps][V], w1[kTaps][V];
#pragma unroll
    for (int j = 0; j < kTaps; ++j) {
        const int src = j - (kTaps - a.taps);
        if (src >= 0) {
            load_f32<T, V>(static_cast<const T *>(a.weight) + src * channels + c0, w0[j]);
            load_f32<T, V>(static_cast<const T *>(a.weight) + src * channels + c1, w1[j]);
        } else {
#pragma unroll
            for (int i = 0; i < V; ++i) w0[j][i] = w1[j][i] = 0.f;
        }
    }

    float h0[kHist > 0 ? kHist : 1][V], h1[kHist > 0 ? kHist : 1][V];   // [b]: the row b + 1 back
    float x0[V], x1[V], n0[V], n1[V];
    load_f32<T, V>(qkv + t0 * a.stride + c0, n0);
    load_f32<T, V>(qkv + t0 * a.stride + c1, n1);
    bool fresh = true;                                    // the history has to be read for this row's sequence
#pragma unroll 4
    for (int t = static_cast<int>(t0); t < t_end; ++t) {
#pragma unroll
        for (int i = 0; i < V; ++i) { x0[i] = n0[i]; x1[i] = n1[i]; }
        if (t + 1 < t_end) {
            load_f32<T, V>(qkv + static_cast<int64_t>(t + 1) * a.stride + c0, n0);
            load_f32<T, V>(qkv + static_cast<int64_t>(t + 1) * a.stride + c1, n1);
        }
        if (!kDecode && t >= row_end) {
            int s = seq;
            while (s + 1 < a.n_seqs && t >= a.cu[s + 1]) ++s;
            enter(s);
            fresh = true;
        }
        if (fresh) {
            const bool have_state = start > 0 && static_cast<uint32_t>(slot_s) < static_cast<uint32_t>(a.state_slots);
#pragma unroll
            for (int b = 0; b < kHist; ++b) {
                const int src = t - (b + 1);              // row b + 1 back, if it belongs to this portion
                const int row_s = a.taps - 1 - (first - src);   // else this row of the carried ones
                if (b + 1 < a.taps && src >= first) {
                    load_f32<T, V>(qkv + src * a.stride + c0, h0[b]);
                    load_f32<T, V>(qkv + src * a.stride + c1, h1[b]);
                } else if (b + 1 < a.taps && have_state && row_s >= 0) {
                    const T *sp = state + (static_cast<int64_t>(slot_s) * (a.taps - 1) + row_s) * channels;
                    load_f32<T, V>(sp + c0, h0[b]);
                    load_f32<T, V>(sp + c1, h1[b]);
                } else {
#pragma unroll
                    for (int i = 0; i < V; ++i) h0[b][i] = h1[b][i] = 0.f;
                }
            }
            fresh = false;
        }
        float y0[V], y1[V];
#pragma unroll
        for (int i = 0; i < V; ++i) {
            y0[i] = w0[kTaps - 1][i] * x0[i];
            y1[i] = w1[kTaps - 1][i] * x1[i];
#pragma unroll
            for (int b = 0; b < kHist; ++b) {
                y0[i] = fmaf(w0[kTaps - 2 - b][i], h0[b][i], y0[i]);
                y1[i] = fmaf(w1[kTaps - 2 - b][i], h1[b][i], y1[i]);
            }
        }
        if (pair) {
            const int pos = min(max(start + (t - first), 0), a.max_position - 1);
            const float *cs = a.rope + static_cast<int64_t>(pos) * (2 * a.half) + ri;
            float c[V], s[V];
            load_f32<float, V>(cs, c);
            load_f32<float, V>(cs + a.half, s);
#pragma unroll
            for (int i = 0; i < V; ++i) {
                const float p = y0[i] * c[i] - y1[i] * s[i];
                y1[i] = y1[i] * c[i] + y0[i] * s[i];
                y0[i] = p;
            }
        }
        if (!is_v && head < a.heads) {
            T *q = static_cast<T *>(a.q_out) + static_cast<int64_t>(t) * a.heads * a.dim + static_cast<int64_t>(head) * a.dim + off;
            store_f32<T, V>(q, y0);
            if (pair) store_f32<T, V>(q + a.half, y1);
        } else {
            const int64_t slot = a.slot_mapping[t];
            if (slot >= 0 && slot < a.num_slots) {
                if (is_v) {
                    store_f32<T, V>(static_cast<T *>(a.v_cache) + (slot * a.kv_heads + head) * a.vdim + off, y0);
                } else {
                    T *k = static_cast<T *>(a.k_cache) + (slot * a.kv_heads + (head - a.heads)) * a.dim + off;
                    store_f32<T, V>(k, y0);
                    if (pair) store_f32<T, V>(k + a.half, y1);
                }
            }
        }
        if (kDecode) {
            if (a.taps > 1 && static_cast<uint32_t>(slot_s) < static_cast<uint32_t>(a.state_slots)) {
                T *sp = state + static_cast<int64_t>(slot_s) * (a.taps - 1) * channels;
#pragma unroll
                for (int b = 0; b < kHist; ++b) {         // the row b back becomes carried row taps - 2 - b
                    if (b > a.taps - 2) continue;
                    const int64_t at = static_cast<int64_t>(a.taps - 2 - b) * channels;
                    if (b == 0) {
                        store_f32<T, V>(sp + at + c0, x0);
                        if (pair) store_f32<T, V>(sp + at + c1, x1);
                    } else {
                        store_f32<T, V>(sp + at + c0, h0[b > 0 ? b - 1 : 0]);
                        if (pair) store_f32<T, V>(sp + at + c1, h1[b > 0 ? b - 1 : 0]);
                    }
                }
            }
        } else {
#pragma unroll
            for (int b = kHist - 1; b >= 0; --b)
#pragma unroll
                for (int i = 0; i < V; ++i) {
                    h0[b][i] = b == 0 ? x0[i] : h0[b > 0 ? b - 1 : 0][i];
                    h1[b][i] = b == 0 ? x1[i] : h1[b > 0 ? b - 1 : 0][i];
                }
        }
    }
}

// One thread per (sequence, channel).  Row r of the carried rows afterwards holds the projected value
// taps - 1 - r positions before the next token; rows older than the portion come from the old rows (always
// a later row than the one being written), rows before the start of the sequence are zero.
template <typename T>
__global__ __launch_bounds__(256) void conv_state_update_kernel(ConvRopeArgs a, int32_t channels) {
    const int c = blockIdx.x * 256 + threadIdx.x;
    const int seq = blockIdx.y;
    if (c >= channels) return;
    const int slot = a.slots_of_seq[seq];
    if (static_cast<uint32_t>(slot) >= static_cast<uint32_t>(a.state_slots)) return;
    const int first = a.cu[seq], rows = a.cu[seq + 1] - first, start = a.klen[seq] - rows;
    if (rows <= 0) return;
    const int keep = a.taps - 1;
    T *sp = static_cast<T *>(a.state) + static_cast<int64_t>(slot) * keep * channels + c;
    const T *qkv = static_cast<const T *>(a.qkv) + c;
    for (int r = 0; r < keep; ++r) {
        const int local = rows - (keep - r);
        T v = Elem<T>::from_f32(0.f);
        if (local >= 0) v = qkv[static_cast<int64_t>(first + local) * a.stride];
        else if (start + local >= 0) v = sp[static_cast<int64_t>(r + rows) * channels];
        sp[static_cast<int64_t>(r) * channels] = v;
    }
}

template <typename T, int V, int kTokens, bool kDecode>
static void launch_conv_rope(const ConvRopeArgs &a, hipStream_t s) {
    const int64_t units = static_cast<int64_t>(a.heads + a.kv_heads) * (a.dim - a.half) / V + static_cast<int64_t>(a.kv_heads) * a.vdim / V;
    const int64_t groups = (a.n + kTokens - 1) / kTokens;
    const dim3 grid(static_cast<uint32_t>((units * groups + 255) / 256)), block(256);
    if (a.taps <= 1) hipLaunchKernelGGL((conv_rope_store_kernel<T, 1, V, kTokens, kDecode>), grid, block, 0, s, a);
    else if (a.taps <= 2) hipLaunchKernelGGL((conv_rope_store_kernel<T, 2, V, kTokens, kDecode>), grid, block, 0, s, a);
    else if (a.taps <= 4) hipLaunchKernelGGL((conv_rope_store_kernel<T, 4, V, kTokens, kDecode>), grid, block, 0, s, a);
    else if (V == 8 || a.taps <= 8) hipLaunchKernelGGL((conv_rope_store_kernel<T, 8, V, kTokens, kDecode>), grid, block, 0, s, a);
    else hipLaunchKernelGGL((conv_rope_store_kernel<T, V == 8 ? 8 : 16, V, kTokens, kDecode>), grid, block, 0, s, a);
}

template <typename T>
static int run_conv_rope(const ConvRopeArgs &a, bool decode, bool vector, hipStream_t s) {
    if (vector) {
        if (decode) launch_conv_rope<T, 8, 1, true>(a, s);
        else if (a.n < 4096) launch_conv_rope<T, 8, 4, false>(a, s);
        else launch_conv_rope<T, 8, 16, false>(a, s);     // enough rows to fill the machine: fewer rows are read twice
    } else {
        if (decode) launch_conv_rope<T, 1, 1, true>(a, s); else launch_conv_rope<T, 1, 4, false>(a, s);
    }
    int rc = launch_status();
    if (rc != NVA_OK || decode || a.taps <= 1) return rc;
    const int32_t channels = (a.heads + a.kv_heads) * a.dim + a.kv_heads * a.vdim;
    hipLaunchKernelGGL((conv_state_update_kernel<T>), dim3((channels + 255) / 256, a.n_seqs), dim3(256), 0, s, a, channels);
    return launch_status();
}

}  // namespace nva

extern "C" int nva_embed_norm(const int64_t *ids, const void *table, float scale, const void *weight, const void *bias,
                              float *residual, void *out, int32_t rows, int32_t width, int32_t vocab, float eps,
                              int32_t dtype, void *stream) {
    using namespace nva;
    if (rows < 0 || width <= 0 || vocab <= 0) return NVA_ERR_BAD_SHAPE;
    if (!known_dtype(dtype)) return NVA_ERR_UNSUPPORTED_GEOMETRY;
    if (rows == 0) return NVA_OK;
    if (!ids || !table || !weight || !bias || !residual || !out) return NVA_ERR_NULL_POINTER;
    NormArgs a{};
    a.ids = ids; a.x = table; a.x_stride = width; a.residual = residual; a.w_next = weight; a.b_next = bias; a.out = out;
    a.rows = rows; a.src_rows = rows; a.width = width; a.vocab = vocab; a.scale = scale; a.eps = eps;
    hipStream_t s = static_cast<hipStream_t>(stream);
    if (dtype == NVA_DTYPE_BF16) launch_norm<bf16_t, true>(a, norm_vector_ok(a), s);
    else launch_norm<float, true>(a, norm_vector_ok(a), s);
    return launch_status();
}

extern "C" int nva_post_add_norm(const void *y, int64_t y_row_stride, float *residual, const void *post_weight,
                                 const void *post_bias, const void *next_weight, const void *next_bias, void *out,
                                 const int32_t *rows_of, int32_t rows, int32_t src_rows, int32_t width, float eps,
                                 int32_t dtype, void *stream) {
    using namespace nva;
    if (rows < 0 || src_rows < 0 || width <= 0) return NVA_ERR_BAD_SHAPE;
    if (!known_dtype(dtype)) return NVA_ERR_UNSUPPORTED_GEOMETRY;
    if (rows == 0) return NVA_OK;
    if (src_rows == 0 || (!rows_of && rows != src_rows)) return NVA_ERR_BAD_SHAPE;
    if (!y || !residual || !post_weight || !post_bias || !next_weight || !next_bias || !out) return NVA_ERR_NULL_POINTER;
    if (y_row_stride < width) return NVA_ERR_BAD_STRIDE;
    NormArgs a{};
    a.x = y; a.x_stride = y_row_stride; a.residual = residual; a.w_post = post_weight; a.b_post = post_bias;
    a.w_next = next_weight; a.b_next = next_bias; a.out = out; a.rows_of = rows_of; a.rows = rows; a.src_rows = src_rows;
    a.width = width; a.eps = eps;
    hipStream_t s = static_cast<hipStream_t>(stream);
    if (dtype == NVA_DTYPE_BF16) launch_norm<bf16_t, false>(a, norm_vector_ok(a), s);
    else launch_norm<float, false>(a, norm_vector_ok(a), s);
    return launch_status();
}

extern "C" int nva_conv_rope_store(const void *qkv, int64_t qkv_row_stride, const void *conv_weight, void *conv_state,
                                   const int32_t *state_slots_of_seq, const int32_t *cu_seqlens_q, const int32_t *seq_lens,
                                   const int32_t *token_seq, const float *rope_cache,
                                   void *q_out, void *k_cache, void *v_cache, const int32_t *slot_mapping,
                                   int64_t num_slots, int32_t n_tokens, int32_t n_seqs, int32_t num_heads,
                                   int32_t num_kv_heads, int32_t qk_dim, int32_t v_dim, int32_t rot_dims, int32_t taps,
                                   int32_t max_position, int32_t num_state_slots, int32_t dtype, void *stream) {
    using namespace nva;
    if (n_tokens < 0 || n_seqs < 0 || num_heads <= 0 || num_kv_heads <= 0 || qk_dim <= 0 || v_dim <= 0 || rot_dims < 0 ||
        rot_dims > qk_dim || num_slots < 0 || num_state_slots < 0 || max_position <= 0 || taps <= 0)
        return NVA_ERR_BAD_SHAPE;
    if (rot_dims % 2 != 0 || taps > 16 || !known_dtype(dtype)) return NVA_ERR_UNSUPPORTED_GEOMETRY;
    if (n_tokens == 0) return NVA_OK;
    const bool decode = cu_seqlens_q == nullptr;
    if (!qkv || !conv_weight || !seq_lens || !q_out || !k_cache || !v_cache || !slot_mapping)
        return NVA_ERR_NULL_POINTER;
    if (taps > 1 && (!conv_state || !state_slots_of_seq)) return NVA_ERR_NULL_POINTER;
    if (rot_dims > 0 && !rope_cache) return NVA_ERR_NULL_POINTER;
    if (!decode && (!token_seq || n_seqs == 0)) return NVA_ERR_NULL_POINTER;
    if (decode && n_seqs != n_tokens) return NVA_ERR_BAD_SHAPE;
    if (n_seqs > 65535) return NVA_ERR_BAD_SHAPE;
    const int64_t channels = static_cast<int64_t>(num_heads + num_kv_heads) * qk_dim + static_cast<int64_t>(num_kv_heads) * v_dim;
    if (qkv_row_stride < channels) return NVA_ERR_BAD_STRIDE;
    if (channels * n_tokens / 256 > 0x7fffffffLL) return NVA_ERR_BAD_SHAPE;
    ConvRopeArgs a{};
    a.qkv = qkv; a.stride = qkv_row_stride; a.weight = conv_weight; a.state = conv_state; a.slots_of_seq = state_slots_of_seq;
    a.cu = cu_seqlens_q; a.klen = seq_lens; a.token_seq = token_seq; a.rope = rope_cache;
    a.q_out = q_out; a.k_cache = k_cache; a.v_cache = v_cache; a.slot_mapping = slot_mapping; a.num_slots = num_slots;
    a.n = n_tokens; a.n_seqs = n_seqs; a.heads = num_heads; a.kv_heads = num_kv_heads; a.dim = qk_dim; a.vdim = v_dim;
    a.half = rot_dims / 2; a.taps = taps; a.max_position = max_position; a.state_slots = num_state_slots;
    const bool vector = taps <= 8 && qk_dim % 8 == 0 && v_dim % 8 == 0 && a.half % 8 == 0 && qkv_row_stride % 8 == 0 && aligned16(qkv) &&
                        aligned16(conv_weight) && aligned16(conv_state) && aligned16(rope_cache) && aligned16(q_out) &&
                        aligned16(k_cache) && aligned16(v_cache);
    hipStream_t s = static_cast<hipStream_t>(stream);
    return dtype == NVA_DTYPE_BF16 ? run_conv_rope<bf16_t>(a, decode, vector, s) : run_conv_rope<float>(a, decode, vector, s);
}
