// Gated linear attention: linear attention whose state decays by a number for every key channel and token.
//
//   z_t = W2 low_t + b                        low_t: a small map of the token's row, made before; z: heads x dim
//   a_t = sigmoid(z_t)^(1/tau)
//   S_t = diag(a_t) S_(t-1) + k_t v_t^T       o_t = S_t^T q_t
//   out_t = o_t / sqrt(mean_v(o_t^2) + eps) * w * silu(gate_t)
//
// A first pass makes the step's decays and writes q (times its scale), k and the decays as 32-bit rows padded to the key size
// that the walk is compiled for (PALM_GLA_DIM: one library for each); the padding's q and k are zero and its decay one.  The
// decay is the exponential of the logarithm of the sigmoid over tau, so that neither a decay near one nor one near zero loses
// its digits.  Where every sequence brings one token the walk's waves make q, k and decays of their head themselves, while the
// state is on its way to the registers, and the first pass is not needed.  The walk over the tokens, and how a long run of them is cut into chunks that run side by side, is
// linear_recurrence.h's.
#include "linear_recurrence.h"

#ifndef PALM_GLA_DIM
#error "compile with -DPALM_GLA_DIM=<padded key size: 32, 64, 128 or 256>"
#endif

PALM_DEFINE_LAST_ERROR()

constexpr int GLA_DIM = PALM_GLA_DIM;
constexpr int GLA_TOKENS = 4;             // tokens a thread of the first pass makes: a weight of W2 is read once for them

__device__ inline float gla_logsigmoid(float z) { return fminf(z, 0.f) - log1pf(expf(-fabsf(z))); }

// A thread per (head, padded key channel), for GLA_TOKENS tokens.  w2: [rank, heads * dim], the transpose of the matrix as a
// checkpoint stores it, so that neighbouring threads read neighbouring weights.
template <typename T>
__global__ __launch_bounds__(256) void gla_prep_kernel(const T* __restrict__ rows, int row_stride, int q_off, int k_off, float q_scale,
                                                       const float* __restrict__ low, int low_stride, const float* __restrict__ w2,
                                                       const float* __restrict__ bias, int rank, float inv_tau, int n_tokens, int heads,
                                                       int dim, float* __restrict__ prep) {
    const int col = blockIdx.x * blockDim.x + threadIdx.x;
    if (col >= heads * GLA_DIM) return;
    const int h = col / GLA_DIM, d = col % GLA_DIM;
    const int t0 = blockIdx.y * GLA_TOKENS, tt = min(GLA_TOKENS, n_tokens - t0);
    const bool in = d < dim;
    const int channel = h * dim + min(d, dim - 1);
    float z[GLA_TOKENS];
#pragma unroll
    for (int i = 0; i < GLA_TOKENS; ++i) z[i] = bias[channel];
#pragma unroll 4
    for (int r = 0; r < rank; ++r) {
        const float w = w2[(size_t)r * heads * dim + channel];
#pragma unroll
        for (int i = 0; i < GLA_TOKENS; ++i) z[i] = fmaf(low[(size_t)(t0 + min(i, tt - 1)) * low_stride + r], w, z[i]);
    }
#pragma unroll
    for (int i = 0; i < GLA_TOKENS; ++i) {
        if (i >= tt) break;
        const size_t row = (size_t)(t0 + i);
        const T* src = rows + row * row_stride;
        float* o = prep + ((row * heads + h) * 3) * GLA_DIM + d;
        o[0] = in ? to_float(src[q_off + channel]) * q_scale : 0.f;
        o[GLA_DIM] = in ? to_float(src[k_off + channel]) : 0.f;
        o[2 * GLA_DIM] = in ? expf(gla_logsigmoid(z[i]) * inv_tau) : 1.f;
    }
}

// A step of single tokens: a lane makes its key channels' q, k and decay.
template <typename T>
struct GlaDirect {
    static constexpr bool SINGLE = true;
    static constexpr int QREGS = (GLA_DIM + WAVE - 1) / WAVE;
    const T* rows;
    const float* low;
    const float* w2;
    const float* bias;
    int row_stride, q_off, k_off, low_stride, rank, heads, dim;
    float q_scale, inv_tau;
    __device__ void read(size_t row, int h, int lane, float (&in)[3][QREGS]) const {
        const T* __restrict__ src = rows + row * row_stride;
        const float* __restrict__ lo = low + row * low_stride;
        const float* __restrict__ w = w2;
        int channel[QREGS];
        float z[QREGS];
#pragma unroll
        for (int c = 0; c < QREGS; ++c) {
            channel[c] = h * dim + min(c * WAVE + lane, dim - 1);
            z[c] = bias[channel[c]];
        }
#pragma unroll 8
        for (int r = 0; r < rank; ++r) {
            const float l = lo[r];
#pragma unroll
            for (int c = 0; c < QREGS; ++c) z[c] = fmaf(l, w[(size_t)r * heads * dim + channel[c]], z[c]);
        }
#pragma unroll
        for (int c = 0; c < QREGS; ++c) {
            const bool there = c * WAVE + lane < dim;
            const float q = to_float(src[q_off + channel[c]]) * q_scale, k = to_float(src[k_off + channel[c]]);
            in[0][c] = there ? q : 0.f;
            in[1][c] = there ? k : 0.f;
            in[2][c] = there ? expf(gla_logsigmoid(z[c]) * inv_tau) : 1.f;
        }
    }
};

PALM_API int palm_gla_pad() { return GLA_DIM; }

// rows [n, row_stride]: q at q_off, k at k_off (heads * dim each), v at v_off, the gate at g_off (heads * vdim each); low float32
// [n, low_stride], `rank` values a token; state float32 [slots, heads, dim, vdim]; norm_w float32 [vdim]; out [n, heads * vdim].
// Room: prep n * heads * 3 * palm_gla_pad() floats (not needed if max_new is one); with chunks (chunk > 0), max_chunks = ceil(max_new / chunk): starts n_seqs *
// max_chunks * heads * dim * vdim floats and chunk_keep n_seqs * max_chunks * heads * dim floats.
PALM_API int palm_gla(hipStream_t stream, const void* rows, int dtype, int row_stride, int q_off, int k_off, int v_off, int g_off,
                      const float* low, int low_stride, const float* w2, const float* bias, int rank, float tau, float q_scale,
                      const float* norm_w, float eps, float* state, const int* seq_slot, const int* seq_new, const int* cu_new, int n_seqs,
                      int heads, int dim, int vdim, void* out, int max_new, int chunk, float* starts, float* chunk_keep, int n_tokens,
                      float* prep) {
    PALM_CHECK(n_seqs >= 0 && n_tokens >= 0 && heads > 0 && dim > 0 && vdim > 0 && rank > 0, "gla: seqs=%d tokens=%d heads=%d dim=%d vdim=%d rank=%d",
               n_seqs, n_tokens, heads, dim, vdim, rank);
    PALM_CHECK(dim <= GLA_DIM && (GLA_DIM == 32 || dim > GLA_DIM / 2), "gla: built for key sizes up to %d, not %d", GLA_DIM, dim);
    PALM_CHECK(vdim <= 1024, "gla: a value size of %d exceeds 1024", vdim);
    PALM_CHECK(tau > 0.f, "gla: tau %g must be positive", (double)tau);
    PALM_CHECK(chunk >= 0 && (chunk == 0 || (starts && chunk_keep && max_new > 0)), "gla: chunks of %d tokens need their starting states", chunk);
    PALM_CHECK(n_tokens == 0 || (rows && low && w2 && bias && norm_w && state && (prep || max_new == 1) && out), "gla: rows, decays' weights and state are needed");
    if (n_seqs == 0 || n_tokens == 0) return 0;
    const int max_chunks = chunk > 0 ? (max_new + chunk - 1) / chunk : 1;
    PALM_CHECK(heads <= 65535 && (long long)n_seqs * max_chunks <= 65535 && n_tokens <= 65535 * GLA_TOKENS,
               "gla: %d heads / %d sequences x %d chunks / %d tokens are more than one launch takes", heads, n_seqs, max_chunks, n_tokens);
    if (max_new == 1) {
        PALM_DTYPE_SWITCH(dtype, T, {
            const GlaDirect<T> direct{(const T*)rows, low, w2, bias, row_stride, q_off, k_off, low_stride, rank, heads, dim, q_scale, 1.0f / tau};
            linear_recurrence_sized<T, GLA_DIM, true>(stream, n_seqs, 1, 0, nullptr, nullptr, (const T*)rows, row_stride, v_off, g_off, direct, nullptr,
                                                      norm_w, eps, state, seq_slot, seq_new, cu_new, heads, dim, vdim, (T*)out, 0, 0, nullptr);
        });
        PALM_LAUNCHED();
        return 0;
    }
    PALM_DTYPE_SWITCH(dtype, T, {
        gla_prep_kernel<T><<<dim3((heads * GLA_DIM + 255) / 256, (n_tokens + GLA_TOKENS - 1) / GLA_TOKENS), 256, 0, stream>>>(
            (const T*)rows, row_stride, q_off, k_off, q_scale, low, low_stride, w2, bias, rank, 1.0f / tau, n_tokens, heads, dim, prep);
        linear_recurrence_sized<T, GLA_DIM, true>(stream, n_seqs, max_new, chunk, starts, chunk_keep, (const T*)rows, row_stride, v_off, g_off,
                                                  PreparedRows<GLA_DIM, 3>{prep, heads}, nullptr, norm_w, eps, state, seq_slot, seq_new, cu_new, heads, dim, vdim, (T*)out, 0, 0,
                                                  nullptr);
    });
    PALM_LAUNCHED();
    return 0;
}
