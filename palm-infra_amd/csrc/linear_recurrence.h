// The walk of a linear recurrence over a matrix per head, shared by the layers whose state decays by one fixed number a head
// (retention.hip) and by one number for every key channel and token (gla.hip).
//
//   S_t = diag(a_t) S_(t-1) + k_t v_t^T      S: [dim, vdim] per sequence and head, 32-bit, kept between steps
//   o_t = S_t^T q_t
//   out_t = o_t / sqrt(mean_v(o_t^2) + eps) * w * silu(gate_t)         (the norm is per head; w [vdim], one for all heads, or none)
//
// One block per (head, sequence), one thread per value dimension v: the thread keeps column v of S in registers and walks over
// the sequence's new tokens.  A token's q and k (and decays) are the same for every thread of the block: each wave reads the
// rows once, one value a lane, and broadcasts value d to all its lanes as a scalar operand of the multiply-adds (no LDS and no
// barrier in the recurrence); the per-token sums of squares over v are reduced a tile of tokens at a time.  A prompt and a single
// token run the same code, so a prompt leaves the state that its tokens one by one leave.
//
// A long run of new tokens would keep only (heads x sequences) blocks busy, one after the other token.  Such a run is
// cut into chunks of `chunk` tokens, and the recurrence's linearity does the rest in three launches:
//   1. every chunk alone from a zero state: its own sum L_c = sum_t (decays after t) k_t v_t^T, and with decays of their own
//      for every token the product of them over the chunk                                        (all chunks at once)
//   2. the chunks' starting states, one after the other: S_(c+1) = decay_c S_c + L_c, S_0 the kept state   (elementwise)
//   3. every chunk from its starting state, now with outputs                                        (all chunks at once)
// The arithmetic of a token is the same in all three; only the order of the 32-bit sums over the past differs.
#pragma once
#include "common.h"

constexpr int REC_TILE = 8;

enum RecurrenceMode : int { REC_WHOLE = 0, REC_LOCAL = 1, REC_FROM_STARTS = 2 };

__device__ inline float rec_silu(float z) { return z / (1.0f + expf(-z)); }

// Where a token's q, k (and decays) come from.  `read` brings the values of lane, lane + 64, .. of a token's row and head into
// in[0 = q, 1 = k, 2 = decay], q and k zero beyond the key size.  PreparedRows: [row][head][0 = q, 1 = k, 2 = decay][DMAX], 32-bit,
// made by a pass before the walk.  A type with SINGLE set serves runs of one token: nothing is read ahead.
template <int DMAX, int PREP>
struct PreparedRows {
    static constexpr bool SINGLE = false;
    static constexpr int QREGS = (DMAX + WAVE - 1) / WAVE;
    const float* rows;
    int heads;
    __device__ void read(size_t row, int h, int lane, float (&in)[PREP][QREGS]) const {
        const float* __restrict__ qr = rows + ((row * heads + h) * PREP) * DMAX;
#pragma unroll
        for (int c = 0; c < QREGS; ++c) {
            const int at = min(c * WAVE + lane, DMAX - 1);             // (a key size of 32: the upper lanes repeat)
#pragma unroll
            for (int i = 0; i < PREP; ++i) in[i][c] = qr[i * DMAX + at];
        }
    }
};

// CHANNEL: every token has a decay for each key channel (the third of its prepared rows), else one fixed decay a head.
// MAXT: the most threads of a block (the value size, rounded up to whole waves): what the compiler may assume when it
// hands out registers.  A thread keeps DMAX values of S; up to 256 threads a block they all stay in registers.
// inputs: q, k and decays.  rows: v at v_off, the gate at g_off.
template <typename T, int DMAX, int MAXT, bool CHANNEL, typename In>
__global__ __launch_bounds__(MAXT) void linear_recurrence_kernel(int mode, int chunk, int max_chunks, float* __restrict__ starts,
                                 float* __restrict__ chunk_keep, const T* __restrict__ rows,
                                 int row_stride, int v_off, int g_off, const In inputs,
                                 const float* __restrict__ decay, const float* __restrict__ norm_w, float eps,
                                 float* __restrict__ state, const int* __restrict__ seq_slot,
                                 const int* __restrict__ seq_new, const int* __restrict__ cu_new,
                                 int heads, int dim, int vdim, T* __restrict__ out, int act, int joined, float* __restrict__ raw) {
    __shared__ float red[REC_TILE][16];
    __shared__ float o_s[REC_TILE][MAXT];
    constexpr int QREGS = (DMAX + WAVE - 1) / WAVE;
    constexpr int PREP = CHANNEL ? 3 : 2;
    const int h = blockIdx.x, b = blockIdx.y / max_chunks, c = blockIdx.y % max_chunks;
    const int v = threadIdx.x;
    const int lane = threadIdx.x % WAVE, wave = threadIdx.x / WAVE, n_waves = blockDim.x / WAVE;
    // this block's run of tokens: the sequence's new ones, or one chunk of them
    const int seq_tokens = seq_new[b];
    if (c * chunk >= seq_tokens) return;
    const int n_new = mode == REC_WHOLE ? seq_tokens : min(chunk, seq_tokens - c * chunk);
    const int row0 = cu_new[b] + (mode == REC_WHOLE ? 0 : c * chunk);
    const bool mine = v < vdim;
    const float g = CHANNEL ? 1.f : decay[h];
    float* sp = mode == REC_WHOLE ? state + (((size_t)seq_slot[b] * heads + h) * dim) * vdim + v
                                  : starts + ((((size_t)b * max_chunks + c) * heads + h) * dim) * vdim + v;

    // the reads are unconditional (of a row and a column that exist) and what does not belong is set to zero after:
    // no branch between them, so that they are all under way at once
    float S[DMAX];
    {
        const float* at = sp - v + min(v, vdim - 1);
        const bool zero = mode == REC_LOCAL || !mine;
        if (dim == DMAX) {                                        // the usual case: every row exists, one stride for all reads
            const size_t stride = (size_t)vdim;
#pragma unroll
            for (int d = 0; d < DMAX; ++d) S[d] = at[d * stride];
            if (zero) {
#pragma unroll
                for (int d = 0; d < DMAX; ++d) S[d] = 0.f;
            }
        } else {
#pragma unroll
            for (int d = 0; d < DMAX; ++d) {
                const float s0 = at[(size_t)min(d, dim - 1) * vdim];
                S[d] = (zero || d >= dim) ? 0.f : s0;
            }
        }
    }

    // A token's inputs: the thread's value, and of the token's q, k (and decay) rows (the same for all threads) one value a
    // lane, which the wave hands to all its lanes as scalars.  The next token's are read while this one's are used.
    const int vc = min(v, vdim - 1);
    auto read_token = [&](int t, float& vv, float (&in)[PREP][QREGS]) {
        const size_t row = (size_t)(row0 + t);
        vv = to_float(rows[row * row_stride + v_off + h * vdim + vc]);
        if (act) vv = rec_silu(vv);
        inputs.read(row, h, lane, in);
    };
    auto from_lane = [](float x, int d) { return __builtin_bit_cast(float, __builtin_amdgcn_readlane(__builtin_bit_cast(int, x), d % WAVE)); };
    float vv, in[PREP][QREGS], kept[QREGS];
#pragma unroll
    for (int i = 0; i < QREGS; ++i) kept[i] = 1.f;
    if (n_new > 0) read_token(0, vv, in);
    for (int t0 = 0; t0 < n_new; t0 += REC_TILE) {
        const int tt = min(REC_TILE, n_new - t0);
        for (int ti = 0; ti < tt; ++ti) {                        // not unrolled: the body is DMAX steps long already
            float vn = vv, next[PREP][QREGS];
            if constexpr (!In::SINGLE) read_token(min(t0 + ti + 1, n_new - 1), vn, next);
            if (!mine) vv = 0.f;
            float acc = 0.f;
#pragma unroll
            for (int d = 0; d < DMAX; ++d) {
                const float qd = from_lane(in[0][d / WAVE], d), kd = from_lane(in[1][d / WAVE], d);
                const float gd = CHANNEL ? from_lane(in[PREP - 1][d / WAVE], d) : g;
                S[d] = fmaf(gd, S[d], kd * vv);
                acc = fmaf(S[d], qd, acc);
            }
            if (CHANNEL) {
#pragma unroll
                for (int i = 0; i < QREGS; ++i) kept[i] *= in[PREP - 1][i];
            }
            if (mode != REC_LOCAL && joined) {
                if (mine) raw[(size_t)(row0 + t0 + ti) * ((size_t)heads * vdim) + h * vdim + v] = acc;
            } else if (mode != REC_LOCAL) {
                o_s[ti][v] = acc;
                const float ss = wave_sum(acc * acc);
                if (lane == 0) red[ti][wave] = ss;
            }
            if constexpr (!In::SINGLE) {
                vv = vn;
#pragma unroll
                for (int i = 0; i < PREP; ++i)
#pragma unroll
                    for (int c = 0; c < QREGS; ++c) in[i][c] = next[i][c];
            }
        }
        if (mode == REC_LOCAL || joined) continue;
        __syncthreads();
        for (int ti = 0; ti < tt; ++ti) {
            float total = 0.f;
            for (int w = 0; w < n_waves; ++w) total += red[ti][w];
            const float inv = 1.0f / sqrtf(total / (float)vdim + eps);
            const size_t row = (size_t)(row0 + t0 + ti);
            const float gate = to_float(rows[row * row_stride + g_off + h * vdim + vc]);
            const float normed = o_s[ti][v] * inv;
            if (mine)
                out[row * ((size_t)heads * vdim) + h * vdim + v] = from_float<T>((norm_w ? normed * norm_w[vc] : normed) * (gate / (1.0f + expf(-gate))));
        }
        __syncthreads();
    }
    if (mine && n_new > 0 && mode != REC_FROM_STARTS) {
        if (dim == DMAX) {
#pragma unroll
            for (int d = 0; d < DMAX; ++d) sp[(size_t)d * vdim] = S[d];
        } else {
#pragma unroll
            for (int d = 0; d < DMAX; ++d)
                if (d < dim) sp[(size_t)d * vdim] = S[d];
        }
    }
    if (CHANNEL && mode == REC_LOCAL && wave == 0) {
#pragma unroll
        for (int i = 0; i < QREGS; ++i) {
            const int d = i * WAVE + lane;
            if (d < dim) chunk_keep[(((size_t)b * max_chunks + c) * heads + h) * dim + d] = kept[i];
        }
    }
}

// Step 2 above: one thread per element of (sequence, head, dim, vdim).  starts[b][c] holds L_c and leaves as S_c.
template <bool CHANNEL>
__global__ void linear_recurrence_starts_kernel(float* __restrict__ starts, const float* __restrict__ chunk_keep, float* __restrict__ state,
                                                const float* __restrict__ decay, const int* __restrict__ seq_slot,
                                                const int* __restrict__ seq_new, int chunk, int max_chunks, int heads, int dim, int vdim) {
    const int per_head = dim * vdim;
    const int e = blockIdx.x * blockDim.x + threadIdx.x, b = blockIdx.y;
    if (e >= heads * per_head) return;
    const int n_new = seq_new[b];
    if (n_new <= 0) return;
    const float g = CHANNEL ? 1.f : decay[e / per_head];
    float* st = state + (size_t)seq_slot[b] * heads * per_head + e;
    float s = *st;
    for (int c = 0; c * chunk < n_new; ++c) {
        float* at = starts + ((size_t)b * max_chunks + c) * heads * per_head + e;
        const float local = *at;
        *at = s;
        const float keep = CHANNEL ? chunk_keep[((size_t)b * max_chunks + c) * heads * dim + e / vdim] : powf(g, (float)min(chunk, n_new - c * chunk));
        s = fmaf(keep, s, local);
    }
    *st = s;
}

// All launches of a step for one padded key size: chunk == 0 walks over every run in one block a head.
template <typename T, int DMAX, bool CHANNEL, typename In>
static void linear_recurrence_sized(hipStream_t stream, int n_seqs, int max_new, int chunk, float* starts, float* chunk_keep, const T* rows,
                                    int row_stride, int v_off, int g_off, const In& inputs, const float* decay, const float* norm_w, float eps,
                                    float* state, const int* seq_slot, const int* seq_new, const int* cu_new, int heads, int dim, int vdim,
                                    T* out, int act, int joined, float* raw) {
    const int threads = (vdim + WAVE - 1) / WAVE * WAVE;
    const int max_chunks = chunk > 0 ? (max_new + chunk - 1) / chunk : 1;
    const dim3 grid(heads, n_seqs * max_chunks);
    auto walk = [&](int mode) {
        const int run = chunk > 0 ? chunk : 1 << 30;
        if (threads <= 256)
            linear_recurrence_kernel<T, DMAX, 256, CHANNEL, In><<<grid, threads, 0, stream>>>(mode, run, max_chunks, starts, chunk_keep, rows, row_stride,
                v_off, g_off, inputs, decay, norm_w, eps, state, seq_slot, seq_new, cu_new, heads, dim, vdim, out, act, joined, raw);
        else
            linear_recurrence_kernel<T, DMAX, 1024, CHANNEL, In><<<grid, threads, 0, stream>>>(mode, run, max_chunks, starts, chunk_keep, rows, row_stride,
                v_off, g_off, inputs, decay, norm_w, eps, state, seq_slot, seq_new, cu_new, heads, dim, vdim, out, act, joined, raw);
    };
    if (chunk == 0) {
        walk(REC_WHOLE);
    } else {
        walk(REC_LOCAL);
        linear_recurrence_starts_kernel<CHANNEL><<<dim3((heads * dim * vdim + 255) / 256, n_seqs), 256, 0, stream>>>(
            starts, chunk_keep, state, decay, seq_slot, seq_new, chunk, max_chunks, heads, dim, vdim);
        walk(REC_FROM_STARTS);
    }
}
