// Softmax attention with a sink, a window (or chunks), a distance bias and a gate for prompts on the matrix cores, bfloat16, compiled for one padded
// key size and one padded value size (PALM_SINK_KK: key size / 32 rounded up; PALM_SINK_VT: value size / 16 rounded up).
//
// A block of four waves shares the pages of one key/value head: the waves take up to four of the query heads that read it, or
// runs of queries of one head (a wave: 16 QT queries of one head).  A page of 64 keys goes from memory straight into LDS
// (global_load_lds, the next one on its way while this one is used; two pages there), keys as rows of 16-byte chunks, values
// transposed as they are kept; chunks are permuted by the row so that an operand's reads spread over the banks (the lane that
// fills a place fetches the chunk that belongs there).
//
// For every page a wave computes the transposed scores S^T = K Q^T (keys down, queries across), so that a lane's four results of
// a tile are four keys of ONE query: the softmax statistics of a query then live in the lanes of its column.  Which key is a
// tile's row is free: rows are dealt so that the eight weights a lane holds of 32 keys are neighbouring keys, and then the second
// product O^T += V^T P^T takes them as its B operand as they are, its A operand being one 16-byte read of a value row.
// Scores leave the matrix cores as 32-bit sums; maximum, exponentials (base 2: the scores are scaled by scale * log2 e), sums and
// the gate are 32-bit; the weights are rounded to bfloat16 for the second product, whose sums are 32-bit again.  The sink is a
// key without a value: a query's running maximum starts at the sink's score and its running sum at one.
//
// Keys and values lie in pages as in attention_sink.hip (K [pages, kv_heads, 64, dim], V [pages, kv_heads, vdim, 64]), or in runs
// of pages that follow each other (no page table), a key's row in two parts: columns up to dim1 a head's own, the others the
// same for all heads; the strides say where a page, a head and a row begin.
#include "lds_stage.h"
#include "mfma.h"

#ifndef PALM_SINK_KK
#error "compile with -DPALM_SINK_KK=<ceil(key size / 32)> -DPALM_SINK_VT=<ceil(value size / 16)>"
#endif

PALM_DEFINE_LAST_ERROR()

constexpr int KK = PALM_SINK_KK;
constexpr int VT = PALM_SINK_VT;
constexpr int SM_WAVES = 4;
constexpr int K_CHUNKS = KK * 4;                               // 16-byte chunks of a key's row in LDS
constexpr int K_BYTES = PAGE_TOKENS * K_CHUNKS * 16, V_BYTES = VT * 16 * PAGE_TOKENS * 2, SM_STAGE = K_BYTES + V_BYTES;
constexpr int V_LOADS = V_BYTES / 1024;                        // instructions that bring a page's values (all waves)

PALM_API int palm_sink_attention_mfma_sizes(int which) { return which == 0 ? KK * 32 : which == 1 ? VT * 16 : SM_WAVES; }

struct PromptKeys {
    const bf16_t *k, *k2, *v;                                  // k2: the columns from dim1 on, for all heads (dim1 = dim: none)
    long long k_page, k_head, k2_page, v_page, v_head;         // elements between pages and between heads
    int k_row, k2_row, v_row, dim1;                            // elements between rows
};

// By what a key row's chunks are permuted: of the eight rows that a read of an operand takes at once (rows 8 a + b, b < 4, for
// two neighbouring a), those that begin in the same bank get different places.
__device__ inline int key_swizzle(int row) {
    return KK % 2 == 0 ? (row & 3) | ((row >> 1) & 4) : ((row >> 1) & 1) | ((row >> 2) & 2);
}

__device__ inline bf16x8 load_row8(const bf16_t* row, int col, int dim) {
    // eight values of a row from column `col`; columns beyond `dim` are zero (dim is a multiple of eight).  The read
    // itself is unconditional (of the row's last eight values where the column lies beyond it): no branch around it
    const bf16x8 v = load_bf16x8(row + min(col, dim - 8));
    return col < dim ? v : zero_bf16x8();
}

template <int QT>
__global__ __launch_bounds__(SM_WAVES * WAVE) void sink_attention_mfma_kernel(
    const bf16_t* __restrict__ q, PromptKeys kv, const int* __restrict__ block_table, int max_pages,
    const int* __restrict__ seq_slot, const int* __restrict__ seq_start, const int* __restrict__ seq_new, const int* __restrict__ cu_new,
    int heads, int kv_heads, int heads_a_block, int dim, int vdim, float scale, int window, int chunked,
    const float* __restrict__ slopes, int has_sink, float sink_score, const float* __restrict__ sink_scores,
    const bf16_t* __restrict__ gate, int gate_stride, int gate_per_head, bf16_t* __restrict__ out) {
    __shared__ __attribute__((aligned(1024))) char lds[2 * SM_STAGE];
    const int b = blockIdx.z;
    const int n_new = seq_new[b];
    const int lane = threadIdx.x % WAVE, wave = __builtin_amdgcn_readfirstlane(threadIdx.x / WAVE);
    const int runs = SM_WAVES / heads_a_block;                  // runs of queries in the block
    // the blocks of late queries, which have the most keys before them (without a window), are handed out first
    const int block_q0 = (gridDim.x - 1 - blockIdx.x) * runs * 16 * QT;
    if (block_q0 >= n_new) return;
    const int per_kv = heads / kv_heads, groups = per_kv / heads_a_block;
    const int kvh = blockIdx.y / groups;
    const int h = kvh * per_kv + blockIdx.y % groups * heads_a_block + wave / runs;
    const int q0 = block_q0 + wave % runs * 16 * QT;            // the wave's first query (beyond the run: it only brings pages)
    if (sink_scores) sink_score = sink_scores[h];               // a learned score for each head instead of one for all
    const int r = lane % 16, g = lane / 16;
    const int start = seq_start[b];
    // the first key that a query at a position sees (may lie below zero)
    auto low_of = [&](int pos) { return window <= 0 ? 0 : chunked ? pos - pos % window : pos - window + 1; };
    int qi[QT], qpos[QT], qlow[QT];
#pragma unroll
    for (int t = 0; t < QT; ++t) {
        qi[t] = min(q0 + 16 * t + r, n_new - 1);                // a column beyond the run repeats the last query and stores nothing
        qpos[t] = start + qi[t];
        qlow[t] = low_of(qpos[t]);
    }
    const int seq_last = start + n_new - 1;
    const int first_pos = start + q0, last_pos = start + min(q0 + 16 * QT - 1, n_new - 1);
    const int last_low = low_of(last_pos);                      // the first key that all of the wave's queries could see
    // the wave's pages and the block's
    const int first_page = max(0, low_of(min(first_pos, seq_last))) / PAGE_TOKENS, last_page = q0 < n_new ? last_pos / PAGE_TOKENS : -1;
    const int block_first = __builtin_amdgcn_readfirstlane(max(0, low_of(start + block_q0)) / PAGE_TOKENS);
    const int block_last = __builtin_amdgcn_readfirstlane((start + min(block_q0 + runs * 16 * QT - 1, n_new - 1)) / PAGE_TOKENS);
    const float log2e = 1.4426950408889634f;
    const float scale2 = scale * log2e;
    const float slope2 = slopes ? slopes[h] * log2e : 0.f;
    const int* pages = block_table ? block_table + (size_t)seq_slot[b] * max_pages : nullptr;
    const int page0 = block_table ? 0 : seq_slot[b];            // without a table: where the sequence's page 0 would lie

    // what this lane brings of every page: instruction i of the block fills 1 KB of the stage
    int k_off[KK];
    bool k_second[KK];
#pragma unroll
    for (int i = 0; i < KK; ++i) {
        const int place = (i * SM_WAVES + wave) * WAVE + lane, row = place / K_CHUNKS;
        const int col = min(((place % K_CHUNKS) ^ key_swizzle(row)) * 8, dim - 8);        // (columns beyond the key meet zeros of the query)
        k_second[i] = col >= kv.dim1;
        k_off[i] = k_second[i] ? row * kv.k2_row + col - kv.dim1 : row * kv.k_row + col;
    }
    constexpr int V_MINE = (V_LOADS + SM_WAVES - 1) / SM_WAVES;
    int v_off[V_MINE];
#pragma unroll
    for (int i = 0; i < V_MINE; ++i) {
        const int place = (i * SM_WAVES + wave) * WAVE + lane, row = place / 8;
        v_off[i] = min(row, vdim - 1) * kv.v_row + ((place % 8) ^ (row & 7)) * 8;
    }
    const uint32_t lds0 = __builtin_amdgcn_readfirstlane((uint32_t)(uintptr_t)(__attribute__((address_space(3))) const void*)lds);
    auto bring = [&](int pg, int stage) {
        const long long page = pages ? pages[pg] : page0 + pg;
        const bf16_t* kp = kv.k + page * kv.k_page + kvh * kv.k_head;
        const bf16_t* kp2 = kv.k2 + page * kv.k2_page;
        const bf16_t* vp = kv.v + page * kv.v_page + kvh * kv.v_head;
        const uint32_t to = __builtin_amdgcn_readfirstlane(lds0 + stage * SM_STAGE);
#pragma unroll
        for (int i = 0; i < KK; ++i) row_chunk_into_lds((k_second[i] ? kp2 : kp) + k_off[i], to + (i * SM_WAVES + wave) * 1024);
#pragma unroll
        for (int i = 0; i < V_MINE; ++i)
            if (i * SM_WAVES + wave < V_LOADS) row_chunk_into_lds(vp + v_off[i], to + K_BYTES + (i * SM_WAVES + wave) * 1024);
    };

    // the queries, as the B operand: column r, eight values of group g for each step of 32 over the key size
    bf16x8 qf[QT][KK];
#pragma unroll
    for (int t = 0; t < QT; ++t) {
        const bf16_t* qr = q + (((size_t)cu_new[b] + qi[t]) * heads + h) * dim;
#pragma unroll
        for (int kk = 0; kk < KK; ++kk) qf[t][kk] = load_row8(qr, kk * 32 + g * 8, dim);
    }
    f32x4 acc[QT][VT];
#pragma unroll
    for (int t = 0; t < QT; ++t)
#pragma unroll
        for (int vt = 0; vt < VT; ++vt) acc[t][vt] = f32x4{0.f, 0.f, 0.f, 0.f};
    // a query's running sum is kept in parts, one a lane group, added at the end: the sink's one goes to group 0
    float mx[QT], l[QT];
#pragma unroll
    for (int t = 0; t < QT; ++t) { mx[t] = has_sink ? sink_score * log2e : -INFINITY; l[t] = has_sink && g == 0 ? 1.f : 0.f; }
    all_but_the_youngest_have_arrived<0>();                     // (the queries: nothing else of this wave is on its way from here on)
    bring(block_first, 0);
    for (int pg = block_first; pg <= block_last; ++pg) {
        char* page = lds + ((pg - block_first) & 1) * SM_STAGE;
        all_but_the_youngest_have_arrived<0>();
        __syncthreads();                                        // every wave's share of the page; and everyone is done with the one before
        if (pg < block_last) bring(pg + 1, (pg + 1 - block_first) & 1);
        // on the page that holds the sequence's last key the values beyond it are made zero: their weights are zero, but pages are
        // handed out uncleared and zero times a stale NaN is NaN
        const int beyond = seq_last - pg * PAGE_TOKENS;
        if (beyond < PAGE_TOKENS - 1) {
            for (int i = threadIdx.x; i < VT * 16 * 8; i += SM_WAVES * WAVE) {
                const int row = i / 8, key0 = ((i % 8) ^ (row & 7)) * 8;
                bf16_t* at = reinterpret_cast<bf16_t*>(page + K_BYTES) + i * 8;
#pragma unroll
                for (int e = 0; e < 8; ++e)
                    if (key0 + e > beyond) at[e].bits = 0;
            }
            __syncthreads();
        }
        if (pg < first_page || pg > last_page) continue;        // (the same in all lanes of the wave)
        f32x4 s[QT][4];
#pragma unroll
        for (int n = 0; n < 4; ++n) {
            const int row = 32 * (n / 2) + 8 * (r / 4) + 4 * (n & 1) + (r & 3);
            const char* kr = page + row * (K_CHUNKS * 16);
            const int swizzle = key_swizzle(row);
#pragma unroll
            for (int t = 0; t < QT; ++t) s[t][n] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
            for (int kk = 0; kk < KK; ++kk) {
                const bf16x8 kf = *reinterpret_cast<const bf16x8*>(kr + ((4 * kk + g) ^ swizzle) * 16);
#pragma unroll
                for (int t = 0; t < QT; ++t) s[t][n] = mfma_16x16x32(kf, qf[t][kk], s[t][n]);
            }
        }
        // lane (r, g) holds the keys 32 (n / 2) + 8 g + 4 (n % 2) + i of query r; scores in units of log2: a weight is one exp2 away
        // the page reaches beyond some query of the wave, or begins before some query's window does
        const bool edge = pg * PAGE_TOKENS + PAGE_TOKENS - 1 > first_pos || pg * PAGE_TOKENS < last_low;
        bf16x8 pf[QT][2];                                       // the weights as B operands: [query tile][32 keys]
#pragma unroll
        for (int t = 0; t < QT; ++t) {
            float top = -INFINITY;
            if (edge || slopes) {
                // the distance bias: key k of the page lies that far beyond the page's first key's distance
                const float base = slope2 * (float)(pg * PAGE_TOKENS + 8 * g - qpos[t]);
#pragma unroll
                for (int n = 0; n < 4; ++n)
#pragma unroll
                    for (int i = 0; i < 4; ++i) {
                        const int k = 32 * (n / 2) + 4 * (n & 1) + i, j = pg * PAGE_TOKENS + 8 * g + k;
                        s[t][n][i] = (j <= qpos[t] && j >= qlow[t]) ? fmaf(s[t][n][i], scale2, fmaf(slope2, (float)k, base)) : -INFINITY;
                        top = fmaxf(top, s[t][n][i]);
                    }
            } else {
#pragma unroll
                for (int n = 0; n < 4; ++n)
#pragma unroll
                    for (int i = 0; i < 4; ++i) {
                        s[t][n][i] *= scale2;
                        top = fmaxf(top, s[t][n][i]);
                    }
            }
            top = fmaxf(top, __shfl_xor(top, 16, WAVE));
            top = fmaxf(top, __shfl_xor(top, 32, WAVE));
            const float m_new = fmaxf(mx[t], top);
            // a query that has seen no key yet and sees none in this page (it has no sink, and the page lies before its
            // window): nothing is weighed, and no difference of infinities is made
            const float m_ref = m_new == -INFINITY ? 0.f : m_new;
            if (__ballot(m_new > mx[t])) {                      // some query's maximum has risen: what it has so far is taken against the new one
                const float alpha = __builtin_amdgcn_exp2f(mx[t] - m_ref);
                l[t] *= alpha;
#pragma unroll
                for (int vt = 0; vt < VT; ++vt)
#pragma unroll
                    for (int i = 0; i < 4; ++i) acc[t][vt][i] *= alpha;
                mx[t] = m_new;
            }
            float sum = 0.f;
#pragma unroll
            for (int n = 0; n < 4; ++n)
#pragma unroll
                for (int i = 0; i < 4; ++i) {
                    s[t][n][i] = __builtin_amdgcn_exp2f(s[t][n][i] - m_ref);
                    sum += s[t][n][i];
                }
            l[t] += sum;                                        // this lane's part; the groups are added at the end
#pragma unroll
            for (int half = 0; half < 2; ++half)
#pragma unroll
                for (int i = 0; i < 4; ++i) {
                    pf[t][half][i] = (__bf16)s[t][2 * half][i];
                    pf[t][half][4 + i] = (__bf16)s[t][2 * half + 1][i];
                }
        }
        // O^T += V^T P^T: row r of a value tile, the same eight keys of group g as the weights hold
        const char* vr = page + K_BYTES + r * 128;
#pragma unroll
        for (int vt = 0; vt < VT; ++vt)
#pragma unroll
            for (int half = 0; half < 2; ++half) {
                const bf16x8 vf = *reinterpret_cast<const bf16x8*>(vr + vt * 2048 + ((4 * half + g) ^ (r & 7)) * 16);
#pragma unroll
                for (int t = 0; t < QT; ++t) acc[t][vt] = mfma_16x16x32(vf, pf[t][half], acc[t][vt]);
            }
    }
    // lane (r, g) holds value dimensions 16 vt + 4 g + i of query r
#pragma unroll
    for (int t = 0; t < QT; ++t) {
        l[t] += __shfl_xor(l[t], 16, WAVE);
        l[t] += __shfl_xor(l[t], 32, WAVE);
        const float f = 1.0f / l[t];
        if (q0 + 16 * t + r >= n_new) continue;
        const size_t row = (size_t)cu_new[b] + qi[t];
        bf16_t* op = out + (row * heads + h) * vdim;
        const bf16_t* gp = gate && !gate_per_head ? gate + row * gate_stride + (size_t)h * vdim : nullptr;
        // one gate value for the whole head: its sigmoid goes into the factor that divides by the sum
        const float fh = gate && gate_per_head ? f / (1.0f + __expf(-to_float(gate[row * gate_stride + h]))) : f;
#pragma unroll
        for (int vt = 0; vt < VT; ++vt) {
            const int vd = 16 * vt + 4 * g;
            if (vd < vdim) {                                        // vdim is a multiple of four
                float o[4];
#pragma unroll
                for (int i = 0; i < 4; ++i) {
                    o[i] = acc[t][vt][i] * fh;
                    if (gp) o[i] *= 1.0f / (1.0f + __expf(-to_float(gp[vd + i])));
                }
                uint2 w;
                w.x = (uint32_t)f32_to_bf16(o[0]).bits | ((uint32_t)f32_to_bf16(o[1]).bits << 16);
                w.y = (uint32_t)f32_to_bf16(o[2]).bits | ((uint32_t)f32_to_bf16(o[3]).bits << 16);
                *reinterpret_cast<uint2*>(op + vd) = w;
            }
        }
    }
}

static int launch_prompt(hipStream_t stream, const void* q, const PromptKeys& kv, const int* block_table, int max_pages, const int* seq_slot,
                         const int* seq_start, const int* seq_new, const int* cu_new, int n_seqs, int max_new, int heads, int kv_heads, int dim,
                         int vdim, float scale, int window, int chunked, const float* slopes, int has_sink, float sink_score,
                         const float* sink_scores, const void* gate, int gate_stride, int gate_per_head, void* out) {
    PALM_CHECK(n_seqs >= 0 && max_new >= 0 && heads > 0 && kv_heads > 0 && dim > 0 && vdim > 0,
               "sink_attention_mfma: seqs=%d max_new=%d heads=%d kv=%d dim=%d vdim=%d", n_seqs, max_new, heads, kv_heads, dim, vdim);
    PALM_CHECK(heads % kv_heads == 0, "sink_attention_mfma: %d heads are not a multiple of %d kv heads", heads, kv_heads);
    PALM_CHECK(dim % 8 == 0 && dim <= KK * 32 && dim > (KK - 1) * 32, "sink_attention_mfma: built for key sizes %d..%d in steps of 8, not %d",
               (KK - 1) * 32 + 8, KK * 32, dim);
    PALM_CHECK(vdim % 4 == 0 && vdim <= VT * 16 && vdim > (VT - 1) * 16, "sink_attention_mfma: built for value sizes %d..%d in steps of 4, not %d",
               (VT - 1) * 16 + 4, VT * 16, vdim);
    PALM_CHECK(window >= 0, "sink_attention_mfma: window %d", window);
    if (n_seqs == 0 || max_new == 0) return 0;
    const int per_kv = heads / kv_heads, heads_a_block = per_kv % 4 == 0 ? 4 : per_kv % 2 == 0 ? 2 : 1;
    const int rows = heads / heads_a_block;
    PALM_CHECK(rows <= 65535 && n_seqs <= 65535, "sink_attention_mfma: %d heads / %d sequences are more than one launch takes", heads, n_seqs);
    auto tiles = [&](int qt) { const int run = SM_WAVES / heads_a_block * 16 * qt; return (max_new + run - 1) / run; };
    PALM_CHECK((long long)kv.v_row * vdim < (1ll << 31) && (long long)max(kv.k_row, kv.k2_row) * PAGE_TOKENS < (1ll << 31),
               "sink_attention_mfma: rows %d, %d and %d elements apart are beyond this kernel's index range", kv.k_row, kv.k2_row, kv.v_row);
#define SINK_LAUNCH(QT) sink_attention_mfma_kernel<QT><<<dim3(tiles(QT), rows, n_seqs), SM_WAVES * WAVE, 0, stream>>>( \
        (const bf16_t*)q, kv, block_table, max_pages, seq_slot, seq_start, seq_new, cu_new, heads, kv_heads, heads_a_block, dim, vdim, scale, \
        window, chunked, slopes, has_sink, sink_score, sink_scores, (const bf16_t*)gate, gate_stride, gate_per_head, (bf16_t*)out)
    // two tiles of queries a wave feed every fragment that it reads to two products (where a lane's registers hold them); one leaves
    // more blocks where they are few
    if constexpr (KK + VT <= 20) {
        if ((long long)tiles(2) * rows * n_seqs >= 1024) SINK_LAUNCH(2); else SINK_LAUNCH(1);
    } else {
        SINK_LAUNCH(1);
    }
#undef SINK_LAUNCH
    PALM_LAUNCHED();
    return 0;
}

PALM_API int palm_sink_attention_mfma(hipStream_t stream, const void* q, const void* k_cache, const void* v_cache,
                                      const int* block_table, int max_pages, const int* seq_slot, const int* seq_start,
                                      const int* seq_new, const int* cu_new, int n_seqs, int max_new, int heads, int kv_heads,
                                      int dim, int vdim, float scale, int window, int chunked, const float* slopes, int has_sink,
                                      float sink_score, const float* sink_scores, const void* gate, int gate_stride, int gate_per_head, void* out) {
    PALM_CHECK(max_pages > 0 && block_table, "sink_attention_mfma: max_pages %d", max_pages);
    const PromptKeys kv{(const bf16_t*)k_cache, (const bf16_t*)k_cache, (const bf16_t*)v_cache, (long long)kv_heads * PAGE_TOKENS * dim,
                        (long long)PAGE_TOKENS * dim, 0, (long long)kv_heads * vdim * PAGE_TOKENS, (long long)vdim * PAGE_TOKENS, dim, 0, PAGE_TOKENS, dim};
    return launch_prompt(stream, q, kv, block_table, max_pages, seq_slot, seq_start, seq_new, cu_new, n_seqs, max_new, heads, kv_heads, dim, vdim,
                         scale, window, chunked, slopes, has_sink, sink_score, sink_scores, gate, gate_stride, gate_per_head, out);
}

// Keys and values laid out one position after the other instead of in a cache's pages: k [positions, heads * dim1] (a head's own
// columns), k2 [positions, dim - dim1] (the rest, for all heads), vt [heads * vdim, positions].  seq_page0[b]: where sequence b's
// page 0 lies in them, in pages (it may lie before the first one if no query sees that far back).
PALM_API int palm_sink_attention_rows_mfma(hipStream_t stream, const void* q, const void* k, const void* k2, const void* vt, int dim1,
                                           int positions, const int* seq_page0, const int* seq_start, const int* seq_new,
                                           const int* cu_new, int n_seqs, int max_new, int heads, int dim, int vdim, float scale, int window,
                                           const float* sink_scores, const void* gate, int gate_stride, void* out) {
    PALM_CHECK(positions > 0 && positions % PAGE_TOKENS == 0 && dim1 > 0 && dim1 % 8 == 0 && dim1 <= dim, "sink_attention_rows: %d positions (whole "
               "pages), key columns %d of %d a head's own", positions, dim1, dim);
    PALM_CHECK(k && vt && (dim1 == dim || k2) && seq_page0, "sink_attention_rows: keys, values and the sequences' pages are needed");
    const PromptKeys kv{(const bf16_t*)k, (const bf16_t*)(k2 ? k2 : k), (const bf16_t*)vt, (long long)PAGE_TOKENS * heads * dim1, dim1,
                        (long long)PAGE_TOKENS * (dim - dim1), PAGE_TOKENS, (long long)vdim * positions, heads * dim1, dim - dim1, positions, dim1};
    return launch_prompt(stream, q, kv, nullptr, 0, seq_page0, seq_start, seq_new, cu_new, n_seqs, max_new, heads, heads, dim, vdim, scale, window, 0,
                         nullptr, sink_scores != nullptr, 0.f, sink_scores, gate, gate_stride, 1, out);
}
