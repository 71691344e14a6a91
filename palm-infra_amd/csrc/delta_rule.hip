// The gated delta rule with one decay per key channel.
//
// Per sequence and head, S [dim, vdim] in 32-bit, kept between steps; for every token, in this order:
//
//   S <- diag(g_t) S                     g_t[d] = exp(-exp(A_h) * softplus(a_t[h, d] + bias[h, d])): one decay per row of S
//   u_t = beta_t (v_t - S^T k_t)         beta_t = sigmoid(b_t[h]): how much of the error is written
//   S <- S + k_t u_t^T
//   o_t = S^T q_t                        (reads the token's own write)
//   out_t = o_t / sqrt(mean_v(o_t^2) + eps) * w * sigmoid(gate_t)           (w [vdim], shared by the heads)
//
// q and k are unit vectors per head, x / sqrt(sum(x^2) + unit_eps), q also times q_scale; head h reads q/k head
// h / (heads / kv_heads).  Decays, gates, unit vectors, state and sums are 32-bit whatever the run's type.
//
// A first pass makes the unit vectors, decays and write strengths of all the step's tokens (32-bit rows, padded to
// the key size that the walk is compiled for; the padding's q and k are zero and its decay one, so the walk's loops need no
// test).  The walk over the tokens, and how a long run of them is cut into chunks that run side by side, is delta_rule.h's.
#include "delta_rule.h"

// One wave per (token, head).  prep[row][head][0 = q, 1 = k, 2 = g][pad];  beta[row][head].
template <typename T>
__global__ __launch_bounds__(WAVE) void delta_prep_kernel(const T* __restrict__ u, int u_stride, int q_off, int k_off,
                                                          const T* __restrict__ b, int b_stride,
                                                          const float* __restrict__ a, int a_stride,
                                                          const float* __restrict__ a_log, const float* __restrict__ dt_bias,
                                                          float q_scale, float unit_eps, int heads, int kv_heads, int dim, int pad,
                                                          float* __restrict__ prep, float* __restrict__ beta) {
    const size_t row = blockIdx.x;
    const int h = blockIdx.y, lane = threadIdx.x;
    const int kh = h / (heads / kv_heads);
    const T* qr = u + row * u_stride + q_off + kh * dim;
    const T* kr = u + row * u_stride + k_off + kh * dim;
    float qq = 0.f, kk = 0.f;
    for (int d = lane; d < dim; d += WAVE) {
        const float qv = to_float(qr[d]), kv = to_float(kr[d]);
        qq = fmaf(qv, qv, qq);
        kk = fmaf(kv, kv, kk);
    }
    const float qi = q_scale / sqrtf(wave_sum(qq) + unit_eps), ki = 1.0f / sqrtf(wave_sum(kk) + unit_eps);
    const float rate = -expf(a_log[h]);
    float* o = prep + ((row * heads + h) * 3) * pad;
    for (int d = lane; d < pad; d += WAVE) {
        const bool in = d < dim;
        o[d] = in ? to_float(qr[d]) * qi : 0.f;
        o[pad + d] = in ? to_float(kr[d]) * ki : 0.f;
        o[2 * pad + d] = in ? expf(rate * delta_softplus(a[row * a_stride + h * dim + d] + dt_bias[h * dim + d])) : 1.f;
    }
    if (lane == 0) beta[row * heads + h] = delta_sigmoid(to_float(b[row * b_stride + h]));
}

PALM_API int palm_delta_pad(int dim) { return dim <= 32 ? 32 : dim <= 64 ? 64 : dim <= 128 ? 128 : 256; }

// u: the convolution's output [n, u_stride] holding q at q_off (kv_heads * dim), k at k_off, v at v_off (heads * vdim);
// b: the write strengths before the sigmoid, [n, b_stride] of the same type, one a head; a: float32 [n, a_stride], the
// decays' rows before bias and softplus (heads * dim); gate: float32 [n, gate_stride], the output gate before the
// sigmoid (heads * vdim).  prep: room for n * heads * 3 * palm_delta_pad(dim) floats, beta_buf: n * heads floats.
// chunk == 0: every sequence's run in one block per head.  Else, with max_chunks = ceil(max_new / chunk): ext holds
// n_seqs * max_chunks * heads * dim * (vdim + dim) floats and starts n_seqs * max_chunks * heads * dim * vdim.
PALM_API int palm_delta_rule(hipStream_t stream, const void* u, int dtype, int u_stride, int q_off, int k_off, int v_off,
                             const void* b, int b_stride, const float* a, int a_stride, const float* gate, int gate_stride,
                             const float* a_log, const float* dt_bias, const float* norm_w, float q_scale, float unit_eps,
                             float eps, float* state, const int* seq_slot, const int* seq_new, const int* cu_new, int n_seqs,
                             int heads, int kv_heads, int dim, int vdim, void* out, int n_tokens, float* prep, float* beta_buf,
                             int max_new, int chunk, float* ext, float* starts) {
    PALM_CHECK(n_seqs >= 0 && heads > 0 && kv_heads > 0 && dim > 0 && vdim > 0, "delta_rule: seqs=%d heads=%d kv=%d dim=%d vdim=%d",
               n_seqs, heads, kv_heads, dim, vdim);
    PALM_CHECK(heads % kv_heads == 0, "delta_rule: %d heads are not a multiple of %d q/k heads", heads, kv_heads);
    PALM_CHECK(dim <= 256, "delta_rule: a key size of %d exceeds 256", dim);
    PALM_CHECK(vdim <= 1024, "delta_rule: a value size of %d exceeds 1024", vdim);
    PALM_CHECK(n_tokens >= 0 && (n_tokens == 0 || (prep && beta_buf)), "delta_rule: the prepared rows need their room");
    PALM_CHECK(chunk >= 0 && (chunk == 0 || (ext && starts && max_new > 0)), "delta_rule: chunks of %d tokens need room for their sums, "
               "products and starting states", chunk);
    if (n_seqs == 0 || n_tokens == 0) return 0;
    const int max_chunks = chunk > 0 ? (max_new + chunk - 1) / chunk : 1;
    PALM_CHECK(heads <= 65535 && (long long)n_seqs * max_chunks <= 65535, "delta_rule: %d heads / %d sequences x %d chunks are more than one "
               "launch takes", heads, n_seqs, max_chunks);
    const int pad = palm_delta_pad(dim);
#define DELTA_CASE(D) delta_rule_sized<T, T, float, D, false, false>(stream, n_seqs, max_new, chunk, ext, starts, (const T*)u, u_stride, v_off, prep, \
            beta_buf, nullptr, gate, gate_stride, norm_w, eps, state, seq_slot, seq_new, cu_new, heads, kv_heads, dim, vdim, (T*)out)
    PALM_DTYPE_SWITCH(dtype, T, {
        delta_prep_kernel<T><<<dim3(n_tokens, heads), WAVE, 0, stream>>>((const T*)u, u_stride, q_off, k_off, (const T*)b, b_stride, a,
                                                                        a_stride, a_log, dt_bias, q_scale, unit_eps, heads, kv_heads,
                                                                        dim, pad, prep, beta_buf);
        if (pad == 32) DELTA_CASE(32);
        else if (pad == 64) DELTA_CASE(64);
        else if (pad == 128) DELTA_CASE(128);
        else DELTA_CASE(256);
    });
#undef DELTA_CASE
    PALM_LAUNCHED();
    return 0;
}
