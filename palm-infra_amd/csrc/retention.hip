// Retention: linear attention with one fixed decay per head, no softmax and no denominator.
//
//   S_t = g_h S_(t-1) + k_t v_t^T        S: [dim, vdim] per sequence and head, 32-bit, kept between steps
//   o_t = S_t^T q_t
//   out_t = o_t / sqrt(mean_v(o_t^2) + eps) * silu(gate_t)         (the unit norm is per head)
//
// q and k are rotated first (pairs (i, i + rot/2) of the first `rot` dimensions, cos/sin rows of the tokens'
// positions) and k is multiplied by k_scale after the rotation; rotated values, state and sums are 32-bit.
//
// Two options make this the recurrence of other linear attentions as well: `act` puts q, k and v through silu first
// (q and k before the rotation), and `joined` leaves out the per-head unit norm and the gate: the heads' o_t are then
// written as they are, 32-bit, and a pass of its own norms a token's joined heads together, with a weight, and gates
// them (palm_joined_norm_gate).
//
// A first pass rotates q and k of all the step's tokens into 32-bit rows; the walk over the tokens, and how a long run of
// them is cut into chunks that run side by side, is linear_recurrence.h's.
#include "linear_recurrence.h"

// q and k of every token and head, rotated (k also scaled), 32-bit: qk[row][head][0 = q, 1 = k][pad], pad >= dim the
// key size that the main kernel is compiled for; the columns beyond dim are zero, so that the main kernel's loops
// over pad need no test (a zero k leaves its row of S zero, a zero q adds nothing).
template <typename T>
__global__ void retention_rotate_kernel(const T* __restrict__ qkvg, int row_stride, int q_off, int k_off,
                                        const float* __restrict__ cos_t, const float* __restrict__ sin_t, int rot, float k_scale,
                                        int act, int n_tokens, int heads, int dim, int pad, float* __restrict__ qk) {
    const long long idx = (long long)blockIdx.x * blockDim.x + threadIdx.x;
    if (idx >= (long long)n_tokens * heads * pad) return;
    const int d = (int)(idx % pad), h = (int)((idx / pad) % heads);
    const size_t row = (size_t)(idx / ((long long)pad * heads));
    float* o = qk + ((row * heads + h) * 2) * pad + d;
    if (d >= dim) { o[0] = 0.f; o[pad] = 0.f; return; }
    const int half = rot / 2;
    const T* qr = qkvg + row * row_stride + q_off + h * dim;
    const T* kr = qkvg + row * row_stride + k_off + h * dim;
    float qv = to_float(qr[d]), kv = to_float(kr[d]);
    if (act) { qv = rec_silu(qv); kv = rec_silu(kv); }
    if (d < rot) {
        const int i = d < half ? d : d - half;
        const float c = cos_t[row * half + i], sn = sin_t[row * half + i];
        const int partner = d < half ? d + half : d - half;
        float qp = to_float(qr[partner]), kp = to_float(kr[partner]);
        if (act) { qp = rec_silu(qp); kp = rec_silu(kp); }
        // the pair (u, w) becomes (u c - w s, w c + u s)
        qv = d < half ? qv * c - qp * sn : qv * c + qp * sn;
        kv = d < half ? kv * c - kp * sn : kv * c + kp * sn;
    }
    o[0] = qv;
    o[pad] = kv * k_scale;
}

// qk: room for n_tokens * heads * 2 * pad floats (the rotated q and k; pad = palm_retention_pad(dim)).  chunk == 0: every sequence's run in one block
// per head.  Else `starts` holds n_seqs * max_chunks * heads * dim * vdim floats, max_chunks = ceil(max_new / chunk).
PALM_API int palm_retention_pad(int dim) { return dim <= 32 ? 32 : dim <= 64 ? 64 : dim <= 128 ? 128 : 256; }

PALM_API int palm_retention(hipStream_t stream, const void* qkvg, int dtype, int row_stride, int q_off, int k_off, int v_off,
                            int g_off, const float* cos_t, const float* sin_t, int rot, const float* decay, float k_scale,
                            float eps, float* state, const int* seq_slot, const int* seq_new, const int* cu_new, int n_seqs,
                            int heads, int dim, int vdim, void* out, int max_new, int chunk, float* starts, int n_tokens,
                            float* qk, int act, int joined, float* raw) {
    PALM_CHECK(n_seqs >= 0 && heads > 0 && dim > 0 && vdim > 0, "retention: seqs=%d heads=%d dim=%d vdim=%d", n_seqs, heads, dim, vdim);
    PALM_CHECK(dim <= 256, "retention: a key size of %d exceeds 256", dim);
    PALM_CHECK(vdim <= 1024, "retention: a value size of %d exceeds 1024", vdim);
    PALM_CHECK(rot >= 0 && rot <= dim && rot % 2 == 0, "retention: %d rotated dimensions of %d", rot, dim);
    PALM_CHECK(rot == 0 || (cos_t && sin_t), "retention: a rotation needs its cos and sin rows");
    PALM_CHECK(chunk >= 0 && (chunk == 0 || (starts && max_new > 0)), "retention: chunks of %d tokens need their starting states", chunk);
    PALM_CHECK(n_tokens >= 0 && (n_tokens == 0 || qk), "retention: the rotated q and k need their room");
    PALM_CHECK(n_tokens == 0 || (joined ? raw != nullptr : out != nullptr), "retention: the outputs need their room (32-bit rows if the heads are normed together later)");
    if (n_seqs == 0 || n_tokens == 0) return 0;
    const int max_chunks = chunk > 0 ? (max_new + chunk - 1) / chunk : 1;
    PALM_CHECK(heads <= 65535 && (long long)n_seqs * max_chunks <= 65535, "retention: %d heads / %d sequences x %d chunks are more than one launch takes",
               heads, n_seqs, max_chunks);
    const int pad = palm_retention_pad(dim);
    const long long rot_threads = (long long)n_tokens * heads * pad;
#define RET_CASE(D) linear_recurrence_sized<T, D, false>(stream, n_seqs, max_new, chunk, starts, nullptr, (const T*)qkvg, row_stride, v_off, g_off, \
            PreparedRows<D, 2>{qk, heads}, \
            decay, nullptr, eps, state, seq_slot, seq_new, cu_new, heads, dim, vdim, (T*)out, act, joined, raw)
    PALM_DTYPE_SWITCH(dtype, T, {
        retention_rotate_kernel<T><<<(unsigned)((rot_threads + 255) / 256), 256, 0, stream>>>((const T*)qkvg, row_stride, q_off, k_off, cos_t,
                                                                                             sin_t, rot, k_scale, act, n_tokens, heads, dim, pad, qk);
        if (pad == 32) RET_CASE(32);
        else if (pad == 64) RET_CASE(64);
        else if (pad == 128) RET_CASE(128);
        else RET_CASE(256);
    });
#undef RET_CASE
    PALM_LAUNCHED();
    return 0;
}

__device__ inline void ret_load4(const float* p, float (&o)[4]) {
    const float4 v = *reinterpret_cast<const float4*>(p);
    o[0] = v.x; o[1] = v.y; o[2] = v.z; o[3] = v.w;
}
__device__ inline void ret_load4(const bf16_t* p, float (&o)[4]) {
    const uint2 v = *reinterpret_cast<const uint2*>(p);
    o[0] = __builtin_bit_cast(float, v.x << 16); o[1] = __builtin_bit_cast(float, v.x & 0xffff0000u);
    o[2] = __builtin_bit_cast(float, v.y << 16); o[3] = __builtin_bit_cast(float, v.y & 0xffff0000u);
}
__device__ inline void ret_store4(float* p, const float (&v)[4]) { *reinterpret_cast<float4*>(p) = make_float4(v[0], v[1], v[2], v[3]); }
__device__ inline void ret_store4(bf16_t* p, const float (&v)[4]) {
    uint2 w;
    w.x = (uint32_t)f32_to_bf16(v[0]).bits | ((uint32_t)f32_to_bf16(v[1]).bits << 16);
    w.y = (uint32_t)f32_to_bf16(v[2]).bits | ((uint32_t)f32_to_bf16(v[3]).bits << 16);
    *reinterpret_cast<uint2*>(p) = w;
}

// ---- the joined heads normed together and gated -------------------------------------------------------------
// out[t] = raw[t] / sqrt(mean(raw[t]^2) + eps) * weight * f(gate[t]) over a token's whole row of `width` values (all
// heads), f = sigmoid (gate_act 1) or silu (gate_act 0).  raw is 32-bit; the gate lies in rows `gate_stride` elements
// apart.  One block per token.
template <typename T>
__global__ __launch_bounds__(1024) void joined_norm_gate_kernel(const float* __restrict__ raw, const float* __restrict__ weight, float eps,
                                                               const T* __restrict__ gate, int gate_stride, int gate_act, int width,
                                                               T* __restrict__ out) {
    __shared__ float scratch[16];
    const size_t t = blockIdx.x;
    const float* r = raw + t * width;
    float ss = 0.f;
    // four values a read where the row and the gate's rows allow
    const bool by_four = width % 4 == 0 && gate_stride % 4 == 0 && (reinterpret_cast<uintptr_t>(gate) % 16) == 0;
    if (by_four) {
        for (int c = threadIdx.x * 4; c < width; c += blockDim.x * 4) {
            const float4 v = *reinterpret_cast<const float4*>(r + c);
            ss += v.x * v.x + v.y * v.y + v.z * v.z + v.w * v.w;
        }
    } else {
        for (int c = threadIdx.x; c < width; c += blockDim.x) { const float v = r[c]; ss += v * v; }
    }
    const float inv = 1.0f / sqrtf(block_sum(ss, scratch) / (float)width + eps);
    auto gated = [&](float o, float w, float g) {
        const float f = gate_act == 1 ? 1.0f / (1.0f + expf(-g)) : g / (1.0f + expf(-g));
        return o * inv * w * f;
    };
    if (by_four) {
        for (int c = threadIdx.x * 4; c < width; c += blockDim.x * 4) {
            const float4 v = *reinterpret_cast<const float4*>(r + c), w = *reinterpret_cast<const float4*>(weight + c);
            float g[4];
            ret_load4(gate + t * gate_stride + c, g);
            const float y[4] = {gated(v.x, w.x, g[0]), gated(v.y, w.y, g[1]), gated(v.z, w.z, g[2]), gated(v.w, w.w, g[3])};
            ret_store4(out + t * width + c, y);
        }
    } else {
        for (int c = threadIdx.x; c < width; c += blockDim.x)
            out[t * width + c] = from_float<T>(gated(r[c], weight[c], to_float(gate[t * gate_stride + c])));
    }
}

PALM_API int palm_joined_norm_gate(hipStream_t stream, const float* raw, const float* weight, float eps, const void* gate, int dtype,
                                   int gate_stride, int gate_act, int n_tokens, int width, void* out) {
    PALM_CHECK(n_tokens >= 0 && width > 0 && gate_stride >= width, "joined_norm_gate: tokens=%d width=%d gate rows %d apart", n_tokens, width, gate_stride);
    PALM_CHECK(gate_act == 0 || gate_act == 1, "joined_norm_gate: gate activation %d is neither silu (0) nor sigmoid (1)", gate_act);
    if (n_tokens == 0) return 0;
    PALM_DTYPE_SWITCH(dtype, T,
        joined_norm_gate_kernel<T><<<n_tokens, n_tokens >= 256 ? 256 : width >= 2048 ? 1024 : width >= 1024 ? 512 : 256, 0, stream>>>(raw, weight, eps, (const T*)gate, gate_stride, gate_act, width, (T*)out));
    PALM_LAUNCHED();
    return 0;
}

PALM_DEFINE_LAST_ERROR()
