// Attention over one compressed row per position on the matrix cores, bfloat16 (prompts here, single tokens further down); compiled for one padded
// row size and one padded latent size (PALM_LAT_KK: (kv_rank + rot_dim) / 32 rounded up; PALM_LAT_VT: kv_rank / 16
// rounded up).
//
// All heads read the same rows, so a wave owns a tile of 16 queries of HT heads and every fragment of a page that it reads
// feeds HT products.  For every page of 64 keys the wave computes the transposed scores S^T = K Q^T (keys down, queries
// across), so that a lane's four results of a tile are four keys of ONE query: the softmax statistics of a query then live
// in the lanes of its column, and the weights are already laid out as the B operand of the second product O^T += C^T P^T,
// whose A operand reads runs of keys from a transposed copy of the latents.  Scores leave the matrix cores as 32-bit sums;
// maximum, exponentials (base 2: the scores are scaled by scale * log2 e) and sums are 32-bit; the weights are rounded to
// bfloat16 for the second product, whose sums are 32-bit again.
//
// rows [pages, 64, kv_rank + rot_dim]: the keys; rows_t [pages, kv_rank, 64]: the latents once more, positions innermost.
// The two have page tables of their own.  q: float32 [n, heads, kv_rank + rot_dim]; out: float32 [n, heads, kv_rank], or,
// with the value matrices uv [heads * vdim, kv_rank] (and the heads' gates before their sigmoid), out_rows bfloat16
// [n, heads * vdim]: head h's sums through U_v,h times sigmoid(gate_h), made from the registers that hold the sums.
#include "mfma.h"

#ifndef PALM_LAT_KK
#error "compile with -DPALM_LAT_KK=<ceil((kv_rank + rot_dim) / 32)> -DPALM_LAT_VT=<ceil(kv_rank / 16)>"
#endif

PALM_DEFINE_LAST_ERROR()

constexpr int KK = PALM_LAT_KK;
constexpr int VT = PALM_LAT_VT;
// heads a wave: as many as a lane's registers take (a head's output tile is 4 VT values a lane, its queries 4 KK)
constexpr int HT = VT <= 8 ? 4 : VT <= 16 ? 2 : 1;

PALM_API int palm_latent_attention_mfma_sizes(int which) { return which == 0 ? KK * 32 : which == 1 ? VT * 16 : HT; }

__device__ inline bf16x8 load_row8(const bf16_t* row, int col, int dim) {
    // eight values of a row from column `col`; columns beyond `dim` are zero (dim is a multiple of eight).  The read
    // itself is unconditional (of the row's last eight values where the column lies beyond it): no branch around it
    const bf16x8 v = load_bf16x8(row + min(col, dim - 8));
    return col < dim ? v : zero_bf16x8();
}

__device__ inline bf16x8 query8(const float* row, int col, int dim) {
    const float* p = row + min(col, dim - 8);
    const float4 a = *reinterpret_cast<const float4*>(p), b = *reinterpret_cast<const float4*>(p + 4);
    bf16x8 v;
    v[0] = (__bf16)a.x; v[1] = (__bf16)a.y; v[2] = (__bf16)a.z; v[3] = (__bf16)a.w;
    v[4] = (__bf16)b.x; v[5] = (__bf16)b.y; v[6] = (__bf16)b.z; v[7] = (__bf16)b.w;
    return col < dim ? v : zero_bf16x8();
}

__global__ __launch_bounds__(WAVE) void latent_attention_mfma_kernel(
    const float* __restrict__ q, const bf16_t* __restrict__ rows, const bf16_t* __restrict__ rows_t,
    const int* __restrict__ block_table, const int* __restrict__ block_table_t, int max_pages,
    const int* __restrict__ seq_slot, const int* __restrict__ seq_start, const int* __restrict__ seq_new,
    const int* __restrict__ cu_new, int heads, int kv_rank, int rot_dim, float scale, int window,
    const float* __restrict__ sink_scores, float* __restrict__ out, const bf16_t* __restrict__ uv, const bf16_t* __restrict__ gate, int gate_stride, int vdim, bf16_t* __restrict__ out_rows) {
    const int h0 = blockIdx.y * HT, b = blockIdx.z;
    const int n_new = seq_new[b];
    const int lane = threadIdx.x;
    // the blocks of late queries, which have the most keys before them, are handed out first
    const int q0 = (gridDim.x - 1 - blockIdx.x) * 16;
    if (q0 >= n_new) return;
    const int r = lane % 16, g = lane / 16;
    const int start = seq_start[b];
    const int dk = kv_rank + rot_dim;
    const int qi = min(q0 + r, n_new - 1);                        // a column beyond the run repeats the last query and stores nothing
    const int qpos = start + qi;
    const int qlo = window > 0 ? max(0, qpos - window + 1) : 0;
    const int last_pos = start + min(q0 + 15, n_new - 1), first_pos = start + q0;
    const int seq_last = start + n_new - 1;                       // rows beyond it belong to nobody
    const float scale2 = scale * 1.4426950408889634f;
    const int* pages = block_table + (size_t)seq_slot[b] * max_pages;
    const int* pages_t = block_table_t + (size_t)seq_slot[b] * max_pages;

    // the queries, as the B operand: column r, eight values of group g for each step of 32 over the row
    bf16x8 qf[HT][KK];
#pragma unroll
    for (int t = 0; t < HT; ++t) {
        const float* qr = q + (((size_t)cu_new[b] + qi) * heads + min(h0 + t, heads - 1)) * dk;
#pragma unroll
        for (int kk = 0; kk < KK; ++kk) qf[t][kk] = query8(qr, kk * 32 + g * 8, dk);
    }
    f32x4 acc[HT][VT];
#pragma unroll
    for (int t = 0; t < HT; ++t)
#pragma unroll
        for (int vt = 0; vt < VT; ++vt) acc[t][vt] = f32x4{0.f, 0.f, 0.f, 0.f};
    float mx[HT], l[HT];
#pragma unroll
    for (int t = 0; t < HT; ++t) {
        // a sink is a key without a value: the running maximum starts at its score, the running sum (lane group 0's part) at one
        mx[t] = sink_scores ? sink_scores[min(h0 + t, heads - 1)] * 1.4426950408889634f : -INFINITY;
        l[t] = sink_scores && g == 0 ? 1.f : 0.f;
    }

    const int first_page = (window > 0 ? max(0, first_pos - window + 1) : 0) / PAGE_TOKENS;
    const int last_page = last_pos / PAGE_TOKENS;
    for (int pg = first_page; pg <= last_page; ++pg) {
        const bf16_t* kp = rows + (size_t)pages[pg] * PAGE_TOKENS * dk;
        const bf16_t* vp = rows_t + (size_t)pages_t[pg] * kv_rank * PAGE_TOKENS;
        f32x4 s[HT][4];
#pragma unroll
        for (int n = 0; n < 4; ++n) {
            bf16x8 kf[KK];
#pragma unroll
            for (int kk = 0; kk < KK; ++kk) kf[kk] = load_row8(kp + (size_t)(16 * n + r) * dk, kk * 32 + g * 8, dk);
#pragma unroll
            for (int t = 0; t < HT; ++t) {
                s[t][n] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
                for (int kk = 0; kk < KK; ++kk) s[t][n] = mfma_16x16x32(kf[kk], qf[t][kk], s[t][n]);
            }
        }
        // lane (r, g) holds the keys 16 n + 4 g + i of query r; scores in units of log2: a weight is one exp2 away
        bf16x8 pf[HT][2];                                          // the weights as B operands: [head][32 keys]
#pragma unroll
        for (int t = 0; t < HT; ++t) {
            float top = -INFINITY;
#pragma unroll
            for (int n = 0; n < 4; ++n)
#pragma unroll
                for (int i = 0; i < 4; ++i) {
                    const int j = pg * PAGE_TOKENS + 16 * n + 4 * g + i;
                    s[t][n][i] = (j <= qpos && j >= qlo) ? s[t][n][i] * scale2 : -INFINITY;     // (a row that belongs to nobody may hold anything)
                    top = fmaxf(top, s[t][n][i]);
                }
            top = fmaxf(top, __shfl_xor(top, 16, WAVE));
            top = fmaxf(top, __shfl_xor(top, 32, WAVE));
            const float m_new = fmaxf(mx[t], top);
            const float m_ref = m_new == -INFINITY ? 0.f : m_new;   // a page of which this query sees nothing yet
            const float alpha = exp2f(mx[t] - m_ref);
            mx[t] = m_new;
            float sum = 0.f;
#pragma unroll
            for (int n = 0; n < 4; ++n)
#pragma unroll
                for (int i = 0; i < 4; ++i) {
                    s[t][n][i] = exp2f(s[t][n][i] - m_ref);
                    sum += s[t][n][i];
                }
            l[t] = l[t] * alpha + sum;                             // this lane's part; the groups are added at the end
#pragma unroll
            for (int vt = 0; vt < VT; ++vt)
#pragma unroll
                for (int i = 0; i < 4; ++i) acc[t][vt][i] *= alpha;
#pragma unroll
            for (int half = 0; half < 2; ++half)
#pragma unroll
                for (int i = 0; i < 4; ++i) {
                    pf[t][half][i] = (__bf16)s[t][2 * half][i];
                    pf[t][half][4 + i] = (__bf16)s[t][2 * half + 1][i];
                }
        }
        // O^T += C^T P^T: row r of a latent tile, the same eight keys of group g as the weights hold.  On the page that
        // holds the sequence's last row the latents of the positions beyond it are taken as zero: their weights are zero,
        // but pages are handed out uncleared and zero times a stale NaN is NaN.
        const int beyond = seq_last - pg * PAGE_TOKENS;            // positions of the page above this belong to nobody
#pragma unroll
        for (int vt = 0; vt < VT; ++vt) {
            const int vd = 16 * vt + r;
            const bf16_t* vr = vp + (size_t)min(vd, kv_rank - 1) * PAGE_TOKENS;
#pragma unroll
            for (int half = 0; half < 2; ++half) {
                const uint2 lo = *reinterpret_cast<const uint2*>(vr + 32 * half + 4 * g);
                const uint2 hi = *reinterpret_cast<const uint2*>(vr + 32 * half + 16 + 4 * g);
                uint32_t w[4] = {lo.x, lo.y, hi.x, hi.y};
                if (beyond < PAGE_TOKENS - 1) {
#pragma unroll
                    for (int e = 0; e < 8; ++e) {
                        const int j = 32 * half + (e < 4 ? 0 : 16) + 4 * g + (e % 4);
                        if (j > beyond) w[e / 2] &= (e % 2) ? 0x0000ffffu : 0xffff0000u;
                    }
                }
                const bf16x8 v8 = vd < kv_rank ? __builtin_bit_cast(bf16x8, make_uint4(w[0], w[1], w[2], w[3])) : zero_bf16x8();
#pragma unroll
                for (int t = 0; t < HT; ++t) acc[t][vt] = mfma_16x16x32(v8, pf[t][half], acc[t][vt]);
            }
        }
    }
    // lane (r, g) holds latent dimensions 16 vt + 4 g + i of query r
#pragma unroll
    for (int t = 0; t < HT; ++t) {
        l[t] += __shfl_xor(l[t], 16, WAVE);
        l[t] += __shfl_xor(l[t], 32, WAVE);
    }
    if (uv) {
        // The value matrix in the same kernel: out^T [vdim, 16 queries] = U_v,h [vdim, kv_rank] (O^T / l).  The sums a lane
        // holds (latent dimensions 16 vt + 4 g + i of query r) are, two tiles at a time, the B operand of a step over 32
        // latent dimensions; the A operand takes the same dimensions of a row of U_v,h.  Then the head's gate.
        constexpr int VP = (VT + 1) / 2;
#pragma unroll
        for (int t = 0; t < HT; ++t) {
            const int h = min(h0 + t, heads - 1);
            const float f = 1.0f / l[t];
            bf16x8 of[VP];
#pragma unroll
            for (int m = 0; m < VP; ++m)
#pragma unroll
                for (int i = 0; i < 4; ++i) {
                    of[m][i] = (__bf16)(acc[t][2 * m][i] * f);
                    of[m][4 + i] = (__bf16)(2 * m + 1 < VT ? acc[t][min(2 * m + 1, VT - 1)][i] * f : 0.f);
                }
            const float gt = gate ? 1.0f / (1.0f + expf(-to_float(gate[((size_t)cu_new[b] + qi) * gate_stride + h]))) : 1.0f;
            for (int j0 = 0; j0 < vdim; j0 += 16) {
                const bf16_t* wr = uv + ((size_t)h * vdim + min(j0 + r, vdim - 1)) * kv_rank;
                f32x4 o = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
                for (int m = 0; m < VP; ++m) {
                    const int k0 = 32 * m + 4 * g, k1 = 32 * m + 16 + 4 * g;          // four dimensions each, inside the latent or beyond it
                    const uint2 lo = *reinterpret_cast<const uint2*>(wr + min(k0, kv_rank - 4));
                    const uint2 hi = *reinterpret_cast<const uint2*>(wr + min(k1, kv_rank - 4));
                    const uint4 both = make_uint4(k0 < kv_rank ? lo.x : 0u, k0 < kv_rank ? lo.y : 0u, k1 < kv_rank ? hi.x : 0u, k1 < kv_rank ? hi.y : 0u);
                    o = mfma_16x16x32(__builtin_bit_cast(bf16x8, both), of[m], o);
                }
                // lane (r, g) holds output dimensions j0 + 4 g + i of query r
                const int j = j0 + 4 * g;
                if (q0 + r < n_new && h0 + t < heads && j < vdim) {                   // vdim is a multiple of four
                    uint2 w;
                    w.x = (uint32_t)f32_to_bf16(o[0] * gt).bits | ((uint32_t)f32_to_bf16(o[1] * gt).bits << 16);
                    w.y = (uint32_t)f32_to_bf16(o[2] * gt).bits | ((uint32_t)f32_to_bf16(o[3] * gt).bits << 16);
                    *reinterpret_cast<uint2*>(out_rows + (((size_t)cu_new[b] + qi) * heads + h0 + t) * vdim + j) = w;
                }
            }
        }
        return;
    }
    if (q0 + r >= n_new) return;
#pragma unroll
    for (int t = 0; t < HT; ++t) {
        if (h0 + t >= heads) continue;
        const float f = 1.0f / l[t];
        float* op = out + (((size_t)cu_new[b] + qi) * heads + h0 + t) * kv_rank;
#pragma unroll
        for (int vt = 0; vt < VT; ++vt) {
            const int vd = 16 * vt + 4 * g;
            if (vd < kv_rank)                                      // kv_rank is a multiple of four
                *reinterpret_cast<float4*>(op + vd) = make_float4(acc[t][vt][0] * f, acc[t][vt][1] * f, acc[t][vt][2] * f, acc[t][vt][3] * f);
        }
    }
}

PALM_API int palm_latent_attention_mfma(hipStream_t stream, const float* q, const void* rows, const void* rows_t,
                                        const int* block_table, const int* block_table_t, int max_pages, const int* seq_slot,
                                        const int* seq_start, const int* seq_new, const int* cu_new, int n_seqs, int max_new,
                                        int heads, int kv_rank, int rot_dim, float scale, int window, const float* sink_scores, float* out,
                                        const void* uv, const void* gate, int gate_stride, int vdim, void* out_rows) {
    PALM_CHECK(n_seqs >= 0 && max_new >= 0 && heads > 0 && kv_rank > 0 && rot_dim >= 0, "latent_attention_mfma: seqs=%d max_new=%d heads=%d "
               "kv_rank=%d rot_dim=%d", n_seqs, max_new, heads, kv_rank, rot_dim);
    const int dk = kv_rank + rot_dim;
    PALM_CHECK(dk % 8 == 0 && dk <= KK * 32 && dk > (KK - 1) * 32, "latent_attention_mfma: built for rows of %d..%d in steps of 8, not %d",
               (KK - 1) * 32 + 8, KK * 32, dk);
    PALM_CHECK(kv_rank % 8 == 0 && kv_rank <= VT * 16 && kv_rank > (VT - 1) * 16, "latent_attention_mfma: built for latents of %d..%d in "
               "steps of 8, not %d", (VT - 1) * 16 + 8, VT * 16, kv_rank);
    PALM_CHECK(window >= 0 && max_pages > 0, "latent_attention_mfma: window %d, max_pages %d", window, max_pages);
    PALM_CHECK(uv ? (out_rows && vdim > 0 && vdim % 4 == 0) : out != nullptr, "latent_attention_mfma: either room for the latent sums, or the "
               "value matrix with room for rows of a value size that is a multiple of four (%d)", vdim);
    if (n_seqs == 0 || max_new == 0) return 0;
    PALM_CHECK(heads <= 65535 * HT && n_seqs <= 65535, "latent_attention_mfma: %d heads / %d sequences are more than one launch takes", heads, n_seqs);
    dim3 grid((max_new + 15) / 16, (heads + HT - 1) / HT, n_seqs);
    latent_attention_mfma_kernel<<<grid, WAVE, 0, stream>>>(q, (const bf16_t*)rows, (const bf16_t*)rows_t, block_table, block_table_t,
                                                           max_pages, seq_slot, seq_start, seq_new, cu_new, heads, kv_rank, rot_dim, scale,
                                                           window, sink_scores, out, (const bf16_t*)uv, (const bf16_t*)gate, gate_stride, vdim,
                                                           (bf16_t*)out_rows);
    PALM_LAUNCHED();
    return 0;
}

// ---- single tokens --------------------------------------------------------------------------------------------------------
// All heads of a token read the same rows, so sixteen heads are the columns of the same two products: a block of four waves
// per (slice of the key range, 16 heads, sequence).  In a page of 64 keys each wave scores sixteen keys (S^T = K Q^T), the page's
// maxima and the weights (bfloat16) cross LDS, and each wave then owns every fourth tile of sixteen latent dimensions of
// O^T += C^T P^T.  The latents of a page are asked for before its scores are made.  A slice leaves its maximum (log2), its sum
// and its unnormalized sums of latents; the merging kernel below adds the sink and applies the value matrices.
constexpr int LD_WAVES = 4;
constexpr int LD_HEADS = 16;
constexpr int LD_TILES = (VT + LD_WAVES - 1) / LD_WAVES;        // latent tiles a wave
constexpr int LD_ROW = PAGE_TOKENS + 8;                         // a head's weights in LDS, padded against bank conflicts

__global__ __launch_bounds__(LD_WAVES * WAVE) void latent_attention_decode_kernel(
    const float* __restrict__ q, const bf16_t* __restrict__ rows, const bf16_t* __restrict__ rows_t,
    const int* __restrict__ block_table, const int* __restrict__ block_table_t, int max_pages,
    const int* __restrict__ seq_slot, const int* __restrict__ seq_start, int heads, int kv_rank, int rot_dim, float scale,
    int window, int n_slices, float* __restrict__ work_ml, float* __restrict__ work) {
    __shared__ float top_s[LD_WAVES][LD_HEADS];
    __shared__ float sum_s[LD_WAVES][LD_HEADS];
    __shared__ __attribute__((aligned(16))) bf16_t p_s[LD_HEADS][LD_ROW];
    const int slice = blockIdx.x, h0 = blockIdx.y * LD_HEADS, b = blockIdx.z;
    const int lane = threadIdx.x % WAVE, wave = threadIdx.x / WAVE;
    const int r = lane % 16, g = lane / 16;
    const int pos = seq_start[b];
    const int lo = window > 0 ? max(0, pos - window + 1) : 0;
    const int dk = kv_rank + rot_dim;
    const float scale2 = scale * 1.4426950408889634f;
    const int* pages = block_table + (size_t)seq_slot[b] * max_pages;
    const int* pages_t = block_table_t + (size_t)seq_slot[b] * max_pages;
    const int p_lo = lo / PAGE_TOKENS, p_hi = pos / PAGE_TOKENS;
    const int per_slice = (p_hi - p_lo + n_slices) / n_slices;
    const int s_lo = p_lo + slice * per_slice, s_hi = min(p_hi, s_lo + per_slice - 1);
    const int head = h0 + r;                                     // the column's head (beyond the last: the last one again, not kept)
    float* ml = work_ml + (((size_t)b * heads + min(head, heads - 1)) * n_slices + slice) * 2;
    if (s_lo > s_hi) {                                           // a slice without pages: the merge reads nothing else of it
        if (wave == 0 && g == 0 && head < heads) { ml[0] = -INFINITY; ml[1] = 0.f; }
        return;
    }

    bf16x8 qf[KK];
    const float* qr = q + ((size_t)b * heads + min(head, heads - 1)) * dk;
#pragma unroll
    for (int kk = 0; kk < KK; ++kk) qf[kk] = query8(qr, kk * 32 + g * 8, dk);
    f32x4 acc[LD_TILES];
#pragma unroll
    for (int i = 0; i < LD_TILES; ++i) acc[i] = f32x4{0.f, 0.f, 0.f, 0.f};
    float mx = -INFINITY, l = 0.f;                               // l: the sum over this lane's keys

    for (int pg = s_lo; pg <= s_hi; ++pg) {
        const bf16_t* kp = rows + ((size_t)pages[pg] * PAGE_TOKENS + 16 * wave + r) * dk;
        const bf16_t* vp = rows_t + (size_t)pages_t[pg] * kv_rank * PAGE_TOKENS;
        bf16x8 kf[KK];
#pragma unroll
        for (int kk = 0; kk < KK; ++kk) kf[kk] = load_bf16x8(kp + min(kk * 32 + g * 8, dk - 8));    // (columns beyond the row meet zeros of the query)
        bf16x8 vf[LD_TILES][2];
#pragma unroll
        for (int i = 0; i < LD_TILES; ++i) {
            const bf16_t* vr = vp + (size_t)min(16 * (wave + LD_WAVES * i) + r, kv_rank - 1) * PAGE_TOKENS;
#pragma unroll
            for (int half = 0; half < 2; ++half) vf[i][half] = load_bf16x8(vr + 32 * half + 8 * g);
        }
        f32x4 s = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int kk = 0; kk < KK; ++kk) s = mfma_16x16x32(kf[kk], qf[kk], s);
        // lane (r, g) holds the keys 16 wave + 4 g + i of head r
        const int j0 = pg * PAGE_TOKENS + 16 * wave + 4 * g;
        float top = -INFINITY;
#pragma unroll
        for (int i = 0; i < 4; ++i) {
            s[i] = (j0 + i <= pos && j0 + i >= lo) ? s[i] * scale2 : -INFINITY;      // (a row that belongs to nobody may hold anything)
            top = fmaxf(top, s[i]);
        }
        top = fmaxf(top, __shfl_xor(top, 16, WAVE));
        top = fmaxf(top, __shfl_xor(top, 32, WAVE));
        if (g == 0) top_s[wave][r] = top;
        __syncthreads();
#pragma unroll
        for (int w = 0; w < LD_WAVES; ++w) top = fmaxf(top, top_s[w][r]);
        const float m_new = fmaxf(mx, top);                      // every page of the range holds a key that is seen: finite
        const float alpha = exp2f(mx - m_new);
        mx = m_new;
        float sum = 0.f;
        bf16_t p[4];
#pragma unroll
        for (int i = 0; i < 4; ++i) {
            const float e = exp2f(s[i] - m_new);
            sum += e;
            p[i] = f32_to_bf16(e);
        }
        l = l * alpha + sum;
        *reinterpret_cast<uint2*>(&p_s[r][16 * wave + 4 * g]) = make_uint2((uint32_t)p[0].bits | ((uint32_t)p[1].bits << 16),
                                                                           (uint32_t)p[2].bits | ((uint32_t)p[3].bits << 16));
        __syncthreads();
        const bf16x8 pf[2] = {load_bf16x8(&p_s[r][8 * g]), load_bf16x8(&p_s[r][32 + 8 * g])};
        // on the page that holds the query's own position the latents beyond it are taken as zero: their weights are zero, but
        // pages are handed out uncleared and zero times a stale NaN is NaN
        const int beyond = pos - pg * PAGE_TOKENS;
        if (beyond < PAGE_TOKENS - 1) {
#pragma unroll
            for (int i = 0; i < LD_TILES; ++i)
#pragma unroll
                for (int half = 0; half < 2; ++half)
#pragma unroll
                    for (int e = 0; e < 8; ++e)
                        if (32 * half + 8 * g + e > beyond) vf[i][half][e] = (__bf16)0.0f;
        }
#pragma unroll
        for (int i = 0; i < LD_TILES; ++i) {
#pragma unroll
            for (int e = 0; e < 4; ++e) acc[i][e] *= alpha;
#pragma unroll
            for (int half = 0; half < 2; ++half) acc[i] = mfma_16x16x32(vf[i][half], pf[half], acc[i]);
        }
    }
    l += __shfl_xor(l, 16, WAVE);
    l += __shfl_xor(l, 32, WAVE);
    if (g == 0) sum_s[wave][r] = l;
    __syncthreads();
    if (head >= heads) return;
    if (wave == 0 && g == 0) {
        float total = 0.f;
#pragma unroll
        for (int w = 0; w < LD_WAVES; ++w) total += sum_s[w][r];
        ml[0] = mx;
        ml[1] = total;
    }
    // lane (r, g) holds latent dimensions 16 tile + 4 g + i of head r
    float* wk = work + (((size_t)b * heads + head) * n_slices + slice) * kv_rank;
#pragma unroll
    for (int i = 0; i < LD_TILES; ++i) {
        const int d = 16 * (wave + LD_WAVES * i) + 4 * g;
        if (d < kv_rank) *reinterpret_cast<float4*>(wk + d) = make_float4(acc[i][0], acc[i][1], acc[i][2], acc[i][3]);
    }
}

// One block per (head, run of LM_ROWS value rows, sequence): the slices of the head merged (with the sink's term in the
// denominator), then out = U_v,h o_lat * sigmoid(gate_h) for its rows.  A wave takes four value rows at a time.
constexpr int LM_WAVES = 4;
constexpr int LM_ROWS = 64;
constexpr int LM_MAX_SLICES = 256;

__global__ __launch_bounds__(LM_WAVES * WAVE) void latent_merge_output_kernel(
    const float* __restrict__ work_ml, const float* __restrict__ work, int n_slices, int heads, int kv_rank,
    const float* __restrict__ sink_scores, const bf16_t* __restrict__ uv, const bf16_t* __restrict__ gate, int gate_stride, int vdim,
    bf16_t* __restrict__ out) {
    __shared__ float w_s[LM_MAX_SLICES];
    __shared__ __attribute__((aligned(16))) float part_s[LM_WAVES][VT * 16];
    __shared__ __attribute__((aligned(16))) float o_s[VT * 16];
    const int h = blockIdx.x, j0 = blockIdx.y * LM_ROWS;
    const size_t b = blockIdx.z;
    const int lane = threadIdx.x % WAVE, wave = threadIdx.x / WAVE;
    const float* ml = work_ml + (b * heads + h) * n_slices * 2;
    float m_all = sink_scores ? sink_scores[h] * 1.4426950408889634f : -INFINITY;
    for (int s = lane; s < n_slices; s += WAVE) m_all = fmaxf(m_all, ml[2 * s]);
    m_all = wave_max(m_all);                                     // (every wave makes it for itself)
    float l = 0.f;
    for (int s = lane; s < n_slices; s += WAVE) {
        const float f = exp2f(ml[2 * s] - m_all);                // a slice without pages: exp2(-inf) = 0
        l = fmaf(ml[2 * s + 1], f, l);
        if (wave == 0) w_s[s] = f;
    }
    l = wave_sum(l);
    if (sink_scores) l += exp2f(sink_scores[h] * 1.4426950408889634f - m_all);
    __syncthreads();
    const float inv = 1.0f / l;
    const float* wk = work + (b * heads + h) * n_slices * kv_rank;
    // a wave takes every fourth slice, a lane four neighbouring columns; what a slice without pages left unwritten counts as nothing
    for (int d = 4 * lane; d < kv_rank; d += 4 * WAVE) {
        float4 o = make_float4(0.f, 0.f, 0.f, 0.f);
#pragma unroll 4
        for (int s = wave; s < n_slices; s += LM_WAVES) {
            const float4 v = *reinterpret_cast<const float4*>(wk + (size_t)s * kv_rank + d);
            const float f = w_s[s];
            o.x = fmaf(f != 0.f ? v.x : 0.f, f, o.x); o.y = fmaf(f != 0.f ? v.y : 0.f, f, o.y);
            o.z = fmaf(f != 0.f ? v.z : 0.f, f, o.z); o.w = fmaf(f != 0.f ? v.w : 0.f, f, o.w);
        }
        *reinterpret_cast<float4*>(&part_s[wave][d]) = o;
    }
    __syncthreads();
    for (int d = threadIdx.x; d < kv_rank; d += LM_WAVES * WAVE) {
        float o = 0.f;
#pragma unroll
        for (int w = 0; w < LM_WAVES; ++w) o += part_s[w][d];
        o_s[d] = o * inv;
    }
    __syncthreads();
    const float gt = gate ? 1.0f / (1.0f + expf(-to_float(gate[b * gate_stride + h]))) : 1.0f;
    for (int j = j0 + 4 * wave; j < min(vdim, j0 + LM_ROWS); j += 4 * LM_WAVES) {
        float acc[4] = {0.f, 0.f, 0.f, 0.f};
        const bf16_t* wr[4];
#pragma unroll
        for (int i = 0; i < 4; ++i) wr[i] = uv + ((size_t)h * vdim + min(j + i, vdim - 1)) * kv_rank;
        for (int d = lane * 8; d < kv_rank; d += WAVE * 8) {
            bf16x8 w8[4];
#pragma unroll
            for (int i = 0; i < 4; ++i) w8[i] = load_bf16x8(wr[i] + d);
#pragma unroll
            for (int e = 0; e < 8; ++e)
#pragma unroll
                for (int i = 0; i < 4; ++i) acc[i] = fmaf((float)w8[i][e], o_s[d + e], acc[i]);
        }
#pragma unroll
        for (int i = 0; i < 4; ++i) {
            const float total = wave_sum(acc[i]);
            if (lane == 0 && j + i < vdim) out[(b * heads + h) * vdim + j + i] = f32_to_bf16(total * gt);
        }
    }
}

// Single tokens of n_seqs sequences.  q float32 [n_seqs, heads, kv_rank + rot_dim]; work_ml: room for n_seqs * heads * n_slices * 2
// floats, work: for n_seqs * heads * n_slices * kv_rank; out bfloat16 [n_seqs, heads * vdim].
PALM_API int palm_latent_attention_decode(hipStream_t stream, const float* q, const void* rows, const void* rows_t,
                                          const int* block_table, const int* block_table_t, int max_pages, const int* seq_slot,
                                          const int* seq_start, int n_seqs, int heads, int kv_rank, int rot_dim, float scale, int window,
                                          const float* sink_scores, int n_slices, float* work_ml, float* work, const void* uv,
                                          const void* gate, int gate_stride, int vdim, void* out) {
    PALM_CHECK(n_seqs >= 0 && heads > 0 && kv_rank > 0 && rot_dim >= 0 && vdim > 0, "latent_attention_decode: seqs=%d heads=%d kv_rank=%d "
               "rot_dim=%d vdim=%d", n_seqs, heads, kv_rank, rot_dim, vdim);
    const int dk = kv_rank + rot_dim;
    PALM_CHECK(dk % 8 == 0 && dk <= KK * 32 && dk > (KK - 1) * 32, "latent_attention_decode: built for rows of %d..%d in steps of 8, not %d",
               (KK - 1) * 32 + 8, KK * 32, dk);
    PALM_CHECK(kv_rank % 8 == 0 && kv_rank <= VT * 16 && kv_rank > (VT - 1) * 16, "latent_attention_decode: built for latents of %d..%d in "
               "steps of 8, not %d", (VT - 1) * 16 + 8, VT * 16, kv_rank);
    PALM_CHECK(window >= 0 && max_pages > 0, "latent_attention_decode: window %d, max_pages %d", window, max_pages);
    PALM_CHECK(n_slices >= 1 && n_slices <= LM_MAX_SLICES && work_ml && work && uv && out, "latent_attention_decode: %d slices (at most %d) need "
               "a workspace, the value matrices and room for the result", n_slices, LM_MAX_SLICES);
    if (n_seqs == 0) return 0;
    const int tiles = (heads + LD_HEADS - 1) / LD_HEADS, runs = (vdim + LM_ROWS - 1) / LM_ROWS;
    PALM_CHECK(tiles <= 65535 && n_seqs <= 65535 && runs <= 65535, "latent_attention_decode: %d heads / %d sequences / a value size of %d are more "
               "than one launch takes", heads, n_seqs, vdim);
    latent_attention_decode_kernel<<<dim3(n_slices, tiles, n_seqs), LD_WAVES * WAVE, 0, stream>>>(
        q, (const bf16_t*)rows, (const bf16_t*)rows_t, block_table, block_table_t, max_pages, seq_slot, seq_start, heads, kv_rank, rot_dim,
        scale, window, n_slices, work_ml, work);
    latent_merge_output_kernel<<<dim3(heads, runs, n_seqs), LM_WAVES * WAVE, 0, stream>>>(
        work_ml, work, n_slices, heads, kv_rank, sink_scores, (const bf16_t*)uv, (const bf16_t*)gate, gate_stride, vdim, (bf16_t*)out);
    PALM_LAUNCHED();
    return 0;
}
