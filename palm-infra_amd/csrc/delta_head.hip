// The gated delta rule with one decay a head, behind short causal convolutions.
//
//   q, k, v   every channel of the projections goes through a causal convolution over time (`taps` taps, the last one the
//             token's own, zeros before the sequence's start) and silu; q and k are then unit vectors per head,
//             x / sqrt(sum(x^2) + unit_eps), q also times q_scale; head h reads q/k head h / (heads / kv_heads)
//   beta_t    sigmoid(b_t[h])
//   g_t       exp(-exp(A_h) softplus(a_t[h] + bias[h])), one number a head
//   S <- g_t S;  u_t = beta_t (v_t - S^T k_t);  S <- S + k_t u_t^T;  o_t = S^T q_t
//   out_t     o_t / sqrt(mean_v(o_t^2) + eps) * w * silu(gate_t)
//
// A first pass does everything before the recurrence: a block per (token, q/k head) with the value heads that read it, so that
// blocks share no channel; convolved values stay 32-bit.  Of the rows before a token's those of its own sequence give the older
// inputs, what lies further back comes from the sequence's kept inputs.  In a step of single tokens the block moves its channels'
// kept inputs on itself; else a second launch does, after all reads.  The walk over the tokens is delta_rule.h's, compiled for
// one padded key size (PALM_DELTA_DIM: one library for each).
#include "conv_state.h"
#include "delta_rule.h"

#ifndef PALM_DELTA_DIM
#error "compile with -DPALM_DELTA_DIM=<padded key size: 32, 64, 128 or 256>"
#endif

PALM_DEFINE_LAST_ERROR()

constexpr int DH_DIM = PALM_DELTA_DIM;
constexpr int DH_THREADS = 256;
constexpr int DH_REGS = (DH_DIM + WAVE - 1) / WAVE;

// rows: q | k | v from column `off` on, channel c of the convolution at column off + c.  ab: float32 rows, b at b_off, a at a_off
// (`heads` values each).  prep[row][q/k head][0 = q, 1 = k][DH_DIM], zero beyond dim; values[row][head][vdim]; beta, decay [row][head].
template <typename T>
__global__ __launch_bounds__(DH_THREADS) void delta_head_prep_kernel(
    const T* __restrict__ rows, int stride, int off, const float* __restrict__ conv_w, int taps, float* __restrict__ conv_state,
    const int* __restrict__ tok_slot, const float* __restrict__ ab, int ab_stride, int b_off, int a_off, const float* __restrict__ a_log,
    const float* __restrict__ dt_bias, float q_scale, float unit_eps, int heads, int kv_heads, int dim, int vdim, int move_state,
    float* __restrict__ prep, float* __restrict__ values, float* __restrict__ beta, float* __restrict__ decay) {
    const size_t t = blockIdx.x;
    const int kh = blockIdx.y, rep = heads / kv_heads;
    const int lane = threadIdx.x % WAVE, wave = threadIdx.x / WAVE;
    const int k0 = kv_heads * dim, v0 = 2 * kv_heads * dim, channels = v0 + heads * vdim;
    const int slot = tok_slot[t];
    float* st = conv_state + (size_t)slot * (taps - 1) * channels;
    int before = 0;                                       // rows right before this one that belong to its sequence (as many as matter)
    while (before < taps - 1 && t > (size_t)before && tok_slot[t - before - 1] == slot) ++before;
    auto convolved = [&](int c) {
        float acc = 0.f;
        for (int j = 0; j < taps; ++j) {
            const int back = taps - 1 - j;
            const float u = back <= before ? to_float(rows[(t - back) * stride + off + c]) : st[(size_t)(taps - 1 - (back - before)) * channels + c];
            acc = fmaf(conv_w[(size_t)c * taps + j], u, acc);
        }
        return acc * delta_sigmoid(acc);
    };
    if (wave < 2) {                                       // wave 0: the q head, wave 1: the k head
        const int c0 = (wave == 0 ? 0 : k0) + kh * dim;
        float x[DH_REGS], ss = 0.f;
#pragma unroll
        for (int i = 0; i < DH_REGS; ++i) {
            const int d = i * WAVE + lane;
            x[i] = d < dim ? convolved(c0 + d) : 0.f;
            ss = fmaf(x[i], x[i], ss);
        }
        const float f = (wave == 0 ? q_scale : 1.0f) / sqrtf(wave_sum(ss) + unit_eps);
        float* o = prep + ((t * kv_heads + kh) * 2 + wave) * DH_DIM;
#pragma unroll
        for (int i = 0; i < DH_REGS; ++i) {
            const int d = i * WAVE + lane;
            if (d < DH_DIM) o[d] = x[i] * f;
        }
    }
    for (int i = threadIdx.x; i < rep * vdim; i += DH_THREADS) {
        const int c = kh * rep * vdim + i;
        values[t * heads * vdim + c] = convolved(v0 + c);
    }
    for (int i = threadIdx.x; i < rep; i += DH_THREADS) {
        const int h = kh * rep + i;
        beta[t * heads + h] = delta_sigmoid(ab[t * ab_stride + b_off + h]);
        decay[t * heads + h] = expf(-expf(a_log[h]) * delta_softplus(ab[t * ab_stride + a_off + h] + dt_bias[h]));
    }
    if (move_state && taps > 1) {
        __syncthreads();                                  // all of the block's reads of its channels' old inputs are done
        for (int i = threadIdx.x; i < 2 * dim + rep * vdim; i += DH_THREADS) {
            const int c = i < dim ? kh * dim + i : i < 2 * dim ? k0 + kh * dim + (i - dim) : v0 + kh * rep * vdim + (i - 2 * dim);
            for (int j = 0; j + 2 < taps; ++j) st[(size_t)j * channels + c] = st[(size_t)(j + 1) * channels + c];
            st[(size_t)(taps - 2) * channels + c] = to_float(rows[t * stride + off + c]);
        }
    }
}

PALM_API int palm_delta_head_pad() { return DH_DIM; }

// rows [n, stride]: q | k | v from column `off`, the gate (heads * vdim) at column g_off; conv_w float32 [channels, taps] and
// conv_state float32 [slots, taps - 1, channels], channels = 2 kv_heads dim + heads vdim; ab float32 [n, ab_stride]; state float32
// [slots, heads, dim, vdim]; norm_w float32 [vdim]; out [n, heads * vdim].  Room: prep n * kv_heads * 2 * palm_delta_head_pad()
// floats, values n * heads * vdim, beta and decay n * heads each; with chunks (chunk > 0), max_chunks = ceil(max_new / chunk):
// ext n_seqs * max_chunks * heads * dim * (vdim + dim) and starts n_seqs * max_chunks * heads * dim * vdim floats.
PALM_API int palm_delta_head(hipStream_t stream, const void* rows, int dtype, int stride, int off, int g_off, const float* conv_w, int taps,
                             float* conv_state, const int* tok_slot, const float* ab, int ab_stride, int b_off, int a_off,
                             const float* a_log, const float* dt_bias, const float* norm_w, float q_scale, float unit_eps, float eps,
                             float* state, const int* seq_slot, const int* seq_new, const int* cu_new, int n_seqs, int n_tokens, int heads,
                             int kv_heads, int dim, int vdim, void* out, float* prep, float* values, float* beta, float* decay, int max_new,
                             int chunk, float* ext, float* starts) {
    PALM_CHECK(n_seqs >= 0 && n_tokens >= 0 && heads > 0 && kv_heads > 0 && dim > 0 && vdim > 0, "delta_head: seqs=%d tokens=%d heads=%d kv=%d dim=%d vdim=%d",
               n_seqs, n_tokens, heads, kv_heads, dim, vdim);
    PALM_CHECK(heads % kv_heads == 0, "delta_head: %d heads are not a multiple of %d q/k heads", heads, kv_heads);
    PALM_CHECK(dim <= DH_DIM && (DH_DIM == 32 || dim > DH_DIM / 2), "delta_head: built for key sizes up to %d, not %d", DH_DIM, dim);
    PALM_CHECK(vdim <= 1024, "delta_head: a value size of %d exceeds 1024", vdim);
    PALM_CHECK(taps >= 1 && taps <= CONV_MAX_TAPS, "delta_head: %d taps (1 to %d)", taps, CONV_MAX_TAPS);
    PALM_CHECK(chunk >= 0 && (chunk == 0 || (ext && starts && max_new > 0)), "delta_head: chunks of %d tokens need room for their sums, products "
               "and starting states", chunk);
    PALM_CHECK(n_tokens == 0 || (rows && conv_w && (taps == 1 || conv_state) && tok_slot && ab && a_log && dt_bias && norm_w && state && prep && values
               && beta && decay && out), "delta_head: rows, weights, states and the prepared rows' room are needed");
    if (n_seqs == 0 || n_tokens == 0) return 0;
    const int max_chunks = chunk > 0 ? (max_new + chunk - 1) / chunk : 1;
    PALM_CHECK(heads <= 65535 && n_seqs <= 65535 && (long long)n_seqs * max_chunks <= 65535, "delta_head: %d heads / %d sequences x %d chunks are more "
               "than one launch takes", heads, n_seqs, max_chunks);
    const int channels = 2 * kv_heads * dim + heads * vdim;
    const int move_state = n_tokens == n_seqs;            // one token a sequence: the pass moves the kept inputs on itself
    PALM_DTYPE_SWITCH(dtype, T, {
        delta_head_prep_kernel<T><<<dim3(n_tokens, kv_heads), DH_THREADS, 0, stream>>>(
            (const T*)rows, stride, off, conv_w, taps, conv_state, tok_slot, ab, ab_stride, b_off, a_off, a_log, dt_bias, q_scale, unit_eps, heads,
            kv_heads, dim, vdim, move_state, prep, values, beta, decay);
        if (taps > 1 && !move_state)
            conv_state_kernel<T><<<dim3((channels + 255) / 256, n_seqs), 256, 0, stream>>>((const T*)rows + off, stride, conv_state, seq_slot, seq_new,
                                                                                          cu_new, channels, taps);
        delta_rule_sized<T, float, T, DH_DIM, true, true>(stream, n_seqs, max_new, chunk, ext, starts, (const float*)values, heads * vdim, 0, prep, beta,
                                                          decay, (const T*)rows + g_off, stride, norm_w, eps, state, seq_slot, seq_new, cu_new, heads,
                                                          kv_heads, dim, vdim, (T*)out);
    });
    PALM_LAUNCHED();
    return 0;
}
