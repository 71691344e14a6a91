// The walk of a gated delta rule, shared by the layers with one decay for every key channel (delta_rule.hip) and with one
// decay a head (delta_head.hip).
//
// Per sequence and head, S [dim, vdim] in 32-bit, kept between steps; for every token, in this order:
//
//   S <- g_t S                           g_t: one number for each row of S, or one for the head
//   u_t = beta_t (v_t - S^T k_t)         beta_t: how much of the error is written
//   S <- S + k_t u_t^T
//   o_t = S^T q_t                        (reads the token's own write)
//   out_t = o_t / sqrt(mean_v(o_t^2) + eps) * w * f(gate_t)           (w [vdim], shared by the heads; f the sigmoid or silu)
//
// One block per (head, sequence), one thread per value dimension v: the columns of S do not depend on each other, so the
// thread keeps column v in registers and walks over the sequence's new tokens.
// A token's q and k (and decays) are the same for every thread of the block: each wave reads the rows once, one value a lane,
// and hands value d to all its lanes as a scalar operand.  A prompt and a single token run the same code, so a
// prompt leaves the state that its tokens one by one leave.
//
// A long run of new tokens would keep only (heads x sequences) blocks busy, one token after the other.  A token's step is
// linear in S: S_t = A_t S_(t-1) + beta_t k_t v_t^T with A_t = (I - beta_t k_t k_t^T) diag(g_t), so such a run is cut into
// chunks of `chunk` tokens and done in three launches:
//   1. every chunk alone: from a zero state with its values (its own sum L_c, [dim, vdim]), and from the identity with
//      values of zero (the product P_c of its A_t, [dim, dim]: the same walk over dim more columns)       (all chunks at once)
//   2. the chunks' starting states, one after the other: S_(c+1) = P_c S_c + L_c, S_0 the kept state      (small products)
//   3. every chunk from its starting state, now with outputs                                             (all chunks at once)
// The arithmetic of a token is the same in all three; only the order of the 32-bit sums over the past differs.
#pragma once
#include "common.h"

constexpr int DELTA_TILE = 8;

__device__ inline float delta_softplus(float z) { return z > 20.f ? z : log1pf(expf(z)); }
__device__ inline float delta_sigmoid(float z) { return 1.0f / (1.0f + expf(-z)); }

enum DeltaMode : int { DELTA_WHOLE = 0, DELTA_LOCAL = 1, DELTA_FROM_STARTS = 2 };

// HEAD_DECAY: one decay for each head and token (decay[row][head]), q and k of a q/k head once for the heads that read it:
// prep[row][q/k head][0 = q, 1 = k][DMAX]; else one decay for each key channel, prep[row][head][0 = q, 1 = k, 2 = g][DMAX].
// values: v of head h at column v_off + h * vdim.  GATE_SILU: the heads' outputs are multiplied by silu of the gate instead of
// its sigmoid.  ext: [sequence x chunk][head][dim][vdim + dim]: a chunk's own sum beside the product of its steps (mode LOCAL writes
// it: blockIdx.z = 0 the value columns, 1 the dim columns that start as the identity).  starts: [sequence x chunk][head]
// [dim][vdim]: the states the chunks start from (mode FROM_STARTS reads them).
template <typename T, typename TV, typename TG, int DMAX, int MAXT, bool HEAD_DECAY, bool GATE_SILU>
__global__ __launch_bounds__(MAXT) void delta_rule_kernel(int mode, int chunk, int max_chunks, float* __restrict__ ext,
                                                          const float* __restrict__ starts,
                                                          const TV* __restrict__ values, int v_stride, int v_off,
                                                          const float* __restrict__ prep, const float* __restrict__ beta,
                                                          const float* __restrict__ decay, const TG* __restrict__ gate, int gate_stride,
                                                          const float* __restrict__ norm_w, float eps,
                                                          float* __restrict__ state, const int* __restrict__ seq_slot,
                                                          const int* __restrict__ seq_new, const int* __restrict__ cu_new,
                                                          int heads, int kv_heads, int dim, int vdim, T* __restrict__ out) {
    __shared__ float red[DELTA_TILE][16];
    __shared__ float o_s[DELTA_TILE][MAXT];
    constexpr int QREGS = (DMAX + WAVE - 1) / WAVE;
    constexpr int PREP = HEAD_DECAY ? 2 : 3;
    const int h = blockIdx.x, b = blockIdx.y / max_chunks, c = blockIdx.y % max_chunks;
    const bool steps_part = blockIdx.z == 1;                     // the columns that become the product of the chunk's steps
    const int v = threadIdx.x;
    const int lane = threadIdx.x % WAVE, wave = threadIdx.x / WAVE, n_waves = blockDim.x / WAVE;
    const int seq_tokens = seq_new[b];
    if (seq_tokens <= 0 || (mode != DELTA_WHOLE && c * chunk >= seq_tokens)) return;
    const int n_new = mode == DELTA_WHOLE ? seq_tokens : min(chunk, seq_tokens - c * chunk);
    const int row0 = cu_new[b] + (mode == DELTA_WHOLE ? 0 : c * chunk);
    const int cols = steps_part ? dim : vdim;
    const bool mine = v < cols;
    const int vc = min(v, vdim - 1);

    // unconditional reads of rows and a column that exist; what does not belong is set to zero after
    float S[DMAX];
    if (mode == DELTA_LOCAL) {
#pragma unroll
        for (int d = 0; d < DMAX; ++d) S[d] = (steps_part && mine && d == v) ? 1.f : 0.f;
    } else {
        const float* sp = mode == DELTA_WHOLE ? state + (((size_t)seq_slot[b] * heads + h) * dim) * vdim + vc
                                              : starts + ((((size_t)b * max_chunks + c) * heads + h) * dim) * vdim + vc;
        if (dim == DMAX) {                                        // the usual case: every row exists, one stride for all reads
            const size_t stride = (size_t)vdim;
#pragma unroll
            for (int d = 0; d < DMAX; ++d) S[d] = sp[d * stride];
            if (!mine) {
#pragma unroll
                for (int d = 0; d < DMAX; ++d) S[d] = 0.f;
            }
        } else {
#pragma unroll
            for (int d = 0; d < DMAX; ++d) {
                const float s0 = sp[(size_t)min(d, dim - 1) * vdim];
                S[d] = (!mine || d >= dim) ? 0.f : s0;
            }
        }
    }

    const int kh = HEAD_DECAY ? h / (heads / kv_heads) : h, prep_heads = HEAD_DECAY ? kv_heads : heads;
    auto read_token = [&](int t, float& vv, float& bt, float& gt, float (&in)[PREP][QREGS]) {
        const size_t row = (size_t)(row0 + t);
        vv = to_float(values[row * v_stride + v_off + h * vdim + vc]);
        bt = beta[row * heads + h];
        gt = HEAD_DECAY ? decay[row * heads + h] : 1.f;
        const float* __restrict__ pr = prep + ((row * prep_heads + kh) * PREP) * DMAX;
#pragma unroll
        for (int c = 0; c < QREGS; ++c) {
            const int at = min(c * WAVE + lane, DMAX - 1);             // (a key size of 32: the upper lanes repeat)
#pragma unroll
            for (int i = 0; i < PREP; ++i) in[i][c] = pr[i * DMAX + at];
        }
    };
    auto from_lane = [](float x, int d) { return __builtin_bit_cast(float, __builtin_amdgcn_readlane(__builtin_bit_cast(int, x), d % WAVE)); };
    float vv, bt, gt, in[PREP][QREGS];
    read_token(0, vv, bt, gt, in);
    for (int t0 = 0; t0 < n_new; t0 += DELTA_TILE) {
        const int tt = min(DELTA_TILE, n_new - t0);
        for (int ti = 0; ti < tt; ++ti) {                        // not unrolled: the body is 2 DMAX steps long already
            float vn, bn, gn, next[PREP][QREGS];
            read_token(min(t0 + ti + 1, n_new - 1), vn, bn, gn, next);
            if (!mine || steps_part) vv = 0.f;
            // four partial sums each: the multiply-adds of a sum over d then wait for every fourth one before them only
            float pr[4] = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
            for (int d = 0; d < DMAX; ++d) {
                const float kd = from_lane(in[1][d / WAVE], d);
                S[d] *= HEAD_DECAY ? gt : from_lane(in[PREP - 1][d / WAVE], d);
                pr[d % 4] = fmaf(S[d], kd, pr[d % 4]);
            }
            const float uu = bt * (vv - ((pr[0] + pr[1]) + (pr[2] + pr[3])));
            float ac[4] = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
            for (int d = 0; d < DMAX; ++d) {
                const float qd = from_lane(in[0][d / WAVE], d), kd = from_lane(in[1][d / WAVE], d);
                S[d] = fmaf(kd, uu, S[d]);
                ac[d % 4] = fmaf(S[d], qd, ac[d % 4]);
            }
            const float acc = (ac[0] + ac[1]) + (ac[2] + ac[3]);
            if (mode != DELTA_LOCAL) {
                o_s[ti][v] = acc;
                const float ss = wave_sum(acc * acc);
                if (lane == 0) red[ti][wave] = ss;
            }
            vv = vn;
            bt = bn;
            gt = gn;
#pragma unroll
            for (int i = 0; i < PREP; ++i)
#pragma unroll
                for (int c = 0; c < QREGS; ++c) in[i][c] = next[i][c];
        }
        if (mode == DELTA_LOCAL) continue;
        __syncthreads();
        for (int ti = 0; ti < tt; ++ti) {
            float total = 0.f;
            for (int w = 0; w < n_waves; ++w) total += red[ti][w];
            const float inv = 1.0f / sqrtf(total / (float)vdim + eps);
            const size_t row = (size_t)(row0 + t0 + ti);
            const float z = to_float(gate[row * gate_stride + h * vdim + vc]);
            const float f = GATE_SILU ? z * delta_sigmoid(z) : delta_sigmoid(z);
            if (mine) out[row * ((size_t)heads * vdim) + h * vdim + v] = from_float<T>((o_s[ti][v] * inv) * norm_w[vc] * f);
        }
        __syncthreads();
    }
    if (mine && mode == DELTA_WHOLE) {
        float* sp = state + (((size_t)seq_slot[b] * heads + h) * dim) * vdim + v;
        if (dim == DMAX) {
#pragma unroll
            for (int d = 0; d < DMAX; ++d) sp[(size_t)d * vdim] = S[d];
        } else {
#pragma unroll
            for (int d = 0; d < DMAX; ++d)
                if (d < dim) sp[(size_t)d * vdim] = S[d];
        }
    }
    if (mine && mode == DELTA_LOCAL) {
        const int ev = vdim + dim;
        float* ep = ext + ((((size_t)b * max_chunks + c) * heads + h) * dim) * ev + (steps_part ? vdim : 0) + v;
#pragma unroll
        for (int d = 0; d < DMAX; ++d)
            if (d < dim) ep[(size_t)d * ev] = S[d];
    }
}

// Step 2 above.  One block per (head, sequence, tile of DS_COLS value columns): the tile of S lies in LDS.  For every chunk
// the block first hands the chunk its starting state, then makes S <- P_c S + L_c: a thread owns one column of the tile and
// every 32nd row of the result (a quarter of a wave a column run, 8 waves x 4 quarters = 32 row groups), reads its rows of
// P_c four values at a time and S from LDS.
constexpr int DS_WAVES = 8;
constexpr int DS_COLS = 16;
constexpr int DS_GROUPS = DS_WAVES * (WAVE / DS_COLS);          // 32 row groups
constexpr int DS_MAX_ROWS = 256 / DS_GROUPS;                    // rows a thread owns at most (dim up to 256)

__global__ __launch_bounds__(DS_WAVES * WAVE) void delta_starts_kernel(const float* __restrict__ ext, float* __restrict__ starts,
                                                                       float* __restrict__ state, const int* __restrict__ seq_slot,
                                                                       const int* __restrict__ seq_new, int chunk, int max_chunks,
                                                                       int heads, int dim, int vdim) {
    extern __shared__ __attribute__((aligned(16))) float s_s[];         // [dim][DS_COLS]
    const int h = blockIdx.x, b = blockIdx.y, v0 = blockIdx.z * DS_COLS;
    const int col = threadIdx.x % DS_COLS, group = threadIdx.x / DS_COLS;
    const int n_new = seq_new[b];
    if (n_new <= 0) return;
    const int v = v0 + col;
    const bool mine = v < vdim;
    const int vc = min(v, vdim - 1), ev = vdim + dim;
    float* st = state + (((size_t)seq_slot[b] * heads + h) * dim) * vdim;
    for (int d = group; d < dim; d += DS_GROUPS) s_s[d * DS_COLS + col] = mine ? st[(size_t)d * vdim + vc] : 0.f;
    __syncthreads();
    for (int c = 0; c * chunk < n_new; ++c) {
        const size_t at = (((size_t)b * max_chunks + c) * heads + h) * dim;
        const float* ep = ext + at * ev;
        float* sc = starts + at * vdim;
        float fresh[DS_MAX_ROWS];
#pragma unroll
        for (int i = 0; i < DS_MAX_ROWS; ++i) {
            const int d = group + i * DS_GROUPS;
            const int dc = min(d, dim - 1);
            const float* pr = ep + (size_t)dc * ev + vdim;              // row d of P_c (16-byte reads where the rows allow them)
            float acc = ep[(size_t)dc * ev + vc];                       // L_c
            if (d < dim) {
                if (ev % 4 == 0 && vdim % 4 == 0 && dim % 4 == 0) {
                    for (int e = 0; e < dim; e += 4) {
                        const float4 p = *reinterpret_cast<const float4*>(pr + e);
                        acc = fmaf(p.x, s_s[e * DS_COLS + col], acc);
                        acc = fmaf(p.y, s_s[(e + 1) * DS_COLS + col], acc);
                        acc = fmaf(p.z, s_s[(e + 2) * DS_COLS + col], acc);
                        acc = fmaf(p.w, s_s[(e + 3) * DS_COLS + col], acc);
                    }
                } else {
                    for (int e = 0; e < dim; ++e) acc = fmaf(pr[e], s_s[e * DS_COLS + col], acc);
                }
            }
            fresh[i] = acc;
        }
        // the chunk starts from the state as it was
        for (int d = group; d < dim; d += DS_GROUPS)
            if (mine) sc[(size_t)d * vdim + v] = s_s[d * DS_COLS + col];
        __syncthreads();
#pragma unroll
        for (int i = 0; i < DS_MAX_ROWS; ++i) {
            const int d = group + i * DS_GROUPS;
            if (d < dim) s_s[d * DS_COLS + col] = fresh[i];
        }
        __syncthreads();
    }
    for (int d = group; d < dim; d += DS_GROUPS)
        if (mine) st[(size_t)d * vdim + v] = s_s[d * DS_COLS + col];
}

// All launches of a step for one padded key size: chunk == 0 walks over every run in one block a head.
template <typename T, typename TV, typename TG, int DMAX, bool HEAD_DECAY, bool GATE_SILU>
static void delta_rule_sized(hipStream_t stream, int n_seqs, int max_new, int chunk, float* ext, float* starts, const TV* values, int v_stride,
                             int v_off, const float* prep, const float* beta, const float* decay, const TG* gate, int gate_stride,
                             const float* norm_w, float eps, float* state, const int* seq_slot, const int* seq_new, const int* cu_new, int heads,
                             int kv_heads, int dim, int vdim, T* out) {
    const int max_chunks = chunk > 0 ? (max_new + chunk - 1) / chunk : 1;
    auto walk = [&](int mode, int parts, int columns) {
        const dim3 grid(heads, n_seqs * max_chunks, parts);
        const int threads = (columns + WAVE - 1) / WAVE * WAVE;
        if (threads <= 256)
            delta_rule_kernel<T, TV, TG, DMAX, 256, HEAD_DECAY, GATE_SILU><<<grid, threads, 0, stream>>>(mode, chunk, max_chunks, ext, starts, values,
                v_stride, v_off, prep, beta, decay, gate, gate_stride, norm_w, eps, state, seq_slot, seq_new, cu_new, heads, kv_heads, dim, vdim, out);
        else
            delta_rule_kernel<T, TV, TG, DMAX, 1024, HEAD_DECAY, GATE_SILU><<<grid, threads, 0, stream>>>(mode, chunk, max_chunks, ext, starts, values,
                v_stride, v_off, prep, beta, decay, gate, gate_stride, norm_w, eps, state, seq_slot, seq_new, cu_new, heads, kv_heads, dim, vdim, out);
    };
    if (chunk == 0) {
        walk(DELTA_WHOLE, 1, vdim);
    } else {
        walk(DELTA_LOCAL, 2, max(vdim, dim));
        delta_starts_kernel<<<dim3(heads, n_seqs, (vdim + DS_COLS - 1) / DS_COLS), DS_WAVES * WAVE, (size_t)dim * DS_COLS * sizeof(float), stream>>>(
            ext, starts, state, seq_slot, seq_new, chunk, max_chunks, heads, dim, vdim);
        walk(DELTA_FROM_STARTS, 1, vdim);
    }
}
