// Routed experts for few rows (a decode step's batch) in bfloat16 on the matrix cores.  Every expert that somebody chose has its
// matrices read once, whatever the number of rows that chose it; nothing is planned on the host and no launch of its own plans.
//
//   up     a block per (expert, run of matrix rows): the block finds the rows that chose its expert (none: it is done), and
//          two waves, half the inner size each, stream 16 rows of the expert's first matrix (gated forms: 16 gate rows and their
//          16 up rows) past them, 16 rows of activations a column tile, and add their sums through LDS; mid[t, c, f] = act(..) in bfloat16, t's choices one after the other, the shared
//          expert's values behind them
//   down   a block per (16 output features, plane): all (row, choice) pairs are sorted by expert in LDS; pieces of 256 inner
//          values of the experts in use are dealt to the planes' waves in turn; a piece's products go, weighted, into the wave's
//          own sums [row, 16 features] in LDS, and the waves' sums are added in their order
//
// A shared expert that every row goes through (weight one, an inner size of its own) runs as one more expert.  Result: float32
// planes [planes, n, width] for a reader that adds them, the first with the rows of other branches.
#include "mfma.h"
#include "expert_form.h"

constexpr int FEW_ROWS = 128;                     // rows of a step at most
constexpr int FEW_UP_WAVES = 4;                   // runs of 16 matrix rows a block, two waves each
constexpr int FEW_DOWN_WAVES = 8;
constexpr int FEW_PIECE = 256;                    // inner values of a piece
constexpr int FEW_STEPS = 8;                      // reads of 32 values of every matrix row under way together
constexpr int FEW_MAX_EXPERTS = 512;
constexpr int FEW_MAX_PAIRS = 4096;

struct FewChoices {
    const int* rows;                 // [n, top], or with ids the table [vocab, top]
    const float* weight;             // [n, top]; null: 1 / top
    const int* ids;
    int vocab, top, n;
    __device__ int expert(int pair) const {
        if (!ids) return rows[pair];
        return rows[(size_t)min(max(ids[pair / top], 0), vocab - 1) * top + pair % top];
    }
};

__device__ inline bf16x8 few_row8(const bf16_t* row, int col, int dim) {
    const bf16x8 v = load_bf16x8(row + min(col, dim - 8));
    return col < dim ? v : zero_bf16x8();
}

// acc[i][ct] += (16 rows of matrix i) x (16 rows of activations in column tile ct) over k0 .. k1 (in steps of eight): lane (r, g) reads row r of each,
// the eight values of group g of every step of 32.  wr: this lane's matrix rows; xr: its activation rows.
template <int MATS, int CT>
__device__ inline void few_products(const bf16_t* const (&wr)[MATS], const bf16_t* const (&xr)[CT], int k0, int k1, int g,
                                    f32x4 (&acc)[MATS][CT]) {
    bf16x8 wf[MATS][FEW_STEPS];
#pragma unroll
    for (int m = 0; m < MATS; ++m)
#pragma unroll
        for (int s = 0; s < FEW_STEPS; ++s) wf[m][s] = few_row8(wr[m], k0 + 32 * s + 8 * g, k1);
    for (int k = k0; k < k1; k += 32 * FEW_STEPS) {
        bf16x8 next[MATS][FEW_STEPS];
        const bool more = k + 32 * FEW_STEPS < k1;
        if (more) {
#pragma unroll
            for (int m = 0; m < MATS; ++m)
#pragma unroll
                for (int s = 0; s < FEW_STEPS; ++s) next[m][s] = few_row8(wr[m], k + 32 * (FEW_STEPS + s) + 8 * g, k1);
        }
#pragma unroll
        for (int s = 0; s < FEW_STEPS; ++s)
#pragma unroll
            for (int ct = 0; ct < CT; ++ct) {
                const bf16x8 xf = few_row8(xr[ct], k + 32 * s + 8 * g, k1);
#pragma unroll
                for (int m = 0; m < MATS; ++m) acc[m][ct] = mfma_16x16x32(wf[m][s], xf, acc[m][ct]);
            }
        if (more) {
#pragma unroll
            for (int m = 0; m < MATS; ++m)
#pragma unroll
                for (int s = 0; s < FEW_STEPS; ++s) wf[m][s] = next[m][s];
        }
    }
}

template <bool GATED, int CT>
__device__ inline void few_up_tile(const bf16_t* __restrict__ h, const bf16_t* __restrict__ w, const int* list, int c0, int m, bool is_shared,
                                   const FewChoices& ch, int width, int ff, int my_ff, int row_ff, int f0, int r, int g, int form,
                                   const ExpertCap& cap, int part, f32x4* exchange, bf16_t* __restrict__ mid) {
    const bf16_t* xr[CT];
    const bf16_t* wr[GATED ? 2 : 1];
#pragma unroll
    for (int ct = 0; ct < CT; ++ct) {
        const int p = list[min(c0 + 16 * ct + r, m - 1)];             // (a column beyond the last repeats it and is not kept)
        xr[ct] = h + (size_t)(is_shared ? p : p / ch.top) * width;
    }
    wr[0] = w + (size_t)min(f0 + r, my_ff - 1) * width;
    if constexpr (GATED) wr[1] = wr[0] + (size_t)my_ff * width;
    f32x4 acc[GATED ? 2 : 1][CT];
#pragma unroll
    for (int i = 0; i < (GATED ? 2 : 1); ++i)
#pragma unroll
        for (int ct = 0; ct < CT; ++ct) acc[i][ct] = f32x4{0.f, 0.f, 0.f, 0.f};
    const int middle = (width / 2 + 31) / 32 * 32;
    if (part == 0) few_products<GATED ? 2 : 1, CT>(wr, xr, 0, min(middle, width), g, acc);
    else if (middle < width) few_products<GATED ? 2 : 1, CT>(wr, xr, middle, width, g, acc);
    __syncthreads();                                                  // (whoever still reads the exchange is done)
    if (part == 1) {
#pragma unroll
        for (int i = 0; i < (GATED ? 2 : 1); ++i)
#pragma unroll
            for (int ct = 0; ct < CT; ++ct) exchange[(i * CT + ct) * WAVE + 16 * g + r] = acc[i][ct];
    }
    __syncthreads();
    if (part == 1) return;
#pragma unroll
    for (int i = 0; i < (GATED ? 2 : 1); ++i)
#pragma unroll
        for (int ct = 0; ct < CT; ++ct) {
            const f32x4 other = exchange[(i * CT + ct) * WAVE + 16 * g + r];
#pragma unroll
            for (int k = 0; k < 4; ++k) acc[i][ct][k] += other[k];
        }
    // lane (r, g) holds inner values f0 + 4 g + i of column r
#pragma unroll
    for (int ct = 0; ct < CT; ++ct) {
        const int col = c0 + 16 * ct + r, f = f0 + 4 * g;
        if (col >= m || f >= my_ff) continue;
        const int p = list[col];
        bf16_t v[4];
#pragma unroll
        for (int i = 0; i < 4; ++i) {
            if constexpr (GATED) v[i] = f32_to_bf16(form == EXPERT_CAPPED ? expert_capped(acc[0][ct][i], acc[1][ct][i], cap) : expert_silu_gated(acc[0][ct][i], acc[1][ct][i]));
            else v[i] = f32_to_bf16(expert_plain(form, acc[0][ct][i]));
        }
        bf16_t* to = mid + (is_shared ? (size_t)p * row_ff + ch.top * ff : (size_t)(p / ch.top) * row_ff + (size_t)(p % ch.top) * ff) + f;
        *reinterpret_cast<uint2*>(to) = make_uint2((uint32_t)v[0].bits | ((uint32_t)v[1].bits << 16), (uint32_t)v[2].bits | ((uint32_t)v[3].bits << 16));
    }
}

template <bool GATED>
__global__ __launch_bounds__(2 * FEW_UP_WAVES * WAVE) void moe_few_up_kernel(const bf16_t* __restrict__ h, const bf16_t* __restrict__ up, FewChoices ch,
                                                                         int experts, int width, int ff, const bf16_t* __restrict__ shared_up,
                                                                         int shared_ff, int form, ExpertCap cap, bf16_t* __restrict__ mid) {
    __shared__ int list_s[FEW_MAX_PAIRS];
    __shared__ int count_s;
    __shared__ f32x4 exchange_s[FEW_UP_WAVES][(GATED ? 2 : 1) * 4 * WAVE];
    const int e = blockIdx.x;
    const bool is_shared = e == experts;
    const int my_ff = is_shared ? shared_ff : ff, row_ff = ch.top * ff + shared_ff;
    const int block_f = blockIdx.y * (16 * FEW_UP_WAVES);
    if (block_f >= my_ff) return;
    if (threadIdx.x == 0) count_s = is_shared ? ch.n : 0;
    __syncthreads();
    if (is_shared) {
        for (int t = threadIdx.x; t < ch.n; t += blockDim.x) list_s[t] = t;
    } else {
        // (the order of the pairs in the list is of no consequence: each is a column of its own)
        for (int p = threadIdx.x; p < ch.n * ch.top; p += blockDim.x)
            if (ch.expert(p) == e) list_s[atomicAdd(&count_s, 1)] = p;
    }
    __syncthreads();
    const int m = count_s;
    const int lane = threadIdx.x % WAVE, wave = threadIdx.x / WAVE % FEW_UP_WAVES, part = threadIdx.x / WAVE / FEW_UP_WAVES;
    const int r = lane % 16, g = lane / 16, f0 = block_f + 16 * wave;   // (rows beyond the matrix: its last one again, not kept)
    if (m == 0) return;
    const bf16_t* w = is_shared ? shared_up : up + (size_t)e * (GATED ? 2 : 1) * ff * width;
    for (int c0 = 0; c0 < m;) {
        const int left = m - c0;
#define FEW_UP(CT) { few_up_tile<GATED, CT>(h, w, list_s, c0, m, is_shared, ch, width, ff, my_ff, row_ff, f0, r, g, form, cap, part, exchange_s[wave], mid); c0 += 16 * CT; }
        if (left > 32) FEW_UP(4) else if (left > 16) FEW_UP(2) else FEW_UP(1)
#undef FEW_UP
    }
}

template <int CT>
__device__ inline void few_down_tile(const bf16_t* __restrict__ mid, const bf16_t* __restrict__ w_row, const int* list, int c0, int m, bool is_shared,
                                     const FewChoices& ch, int ff, int row_ff, int k0, int k1, int r, int g, float* sums) {
    const bf16_t* xr[CT];
    int token[CT];
    float weight[CT];
#pragma unroll
    for (int ct = 0; ct < CT; ++ct) {
        const int col = min(c0 + 16 * ct + r, m - 1);
        const int p = is_shared ? col : list[col];
        token[ct] = is_shared ? p : p / ch.top;
        weight[ct] = is_shared ? 1.0f : ch.weight ? ch.weight[p] : 1.0f / (float)ch.top;
        xr[ct] = mid + (size_t)token[ct] * row_ff + (is_shared ? ch.top * ff : (p % ch.top) * ff);
    }
    const bf16_t* wr[1] = {w_row};
    f32x4 acc[1][CT];
#pragma unroll
    for (int ct = 0; ct < CT; ++ct) acc[0][ct] = f32x4{0.f, 0.f, 0.f, 0.f};
    few_products<1, CT>(wr, xr, k0, k1, g, acc);
    // lane (r, g) holds features 4 g + i of column r; the columns of a tile are different rows
#pragma unroll
    for (int ct = 0; ct < CT; ++ct) {
        if (c0 + 16 * ct + r >= m) continue;
        float4* to = reinterpret_cast<float4*>(sums + token[ct] * 16 + 4 * g);
        float4 v = *to;
        v.x = fmaf(weight[ct], acc[0][ct][0], v.x); v.y = fmaf(weight[ct], acc[0][ct][1], v.y);
        v.z = fmaf(weight[ct], acc[0][ct][2], v.z); v.w = fmaf(weight[ct], acc[0][ct][3], v.w);
        *to = v;
    }
}

__global__ __launch_bounds__(FEW_DOWN_WAVES * WAVE) void moe_few_down_kernel(const bf16_t* __restrict__ mid, const bf16_t* __restrict__ down,
                                                                             FewChoices ch, int experts, int width, int ff,
                                                                             const bf16_t* __restrict__ shared_down, int shared_ff,
                                                                             const bf16_t* __restrict__ add0, const bf16_t* __restrict__ add1,
                                                                             float* __restrict__ out) {
    extern __shared__ __attribute__((aligned(16))) float lds[];
    __shared__ int start_s[FEW_MAX_EXPERTS + 1], cursor_s[FEW_MAX_EXPERTS], used_s[FEW_MAX_EXPERTS];
    __shared__ int n_used_s;
    const int n = ch.n, n_pairs = n * ch.top, row_ff = ch.top * ff + shared_ff;
    float* sums = lds;                                                       // [waves][n][16]
    int* sorted = reinterpret_cast<int*>(lds + FEW_DOWN_WAVES * n * 16);     // [n_pairs]
    const int lane = threadIdx.x % WAVE, wave = threadIdx.x / WAVE;
    const int r = lane % 16, g = lane / 16;
    const int j0 = blockIdx.x * 16, plane = blockIdx.y, planes = gridDim.y;

    for (int e = threadIdx.x; e < experts; e += blockDim.x) cursor_s[e] = 0;
    for (int i = lane; i < n * 16; i += WAVE) sums[wave * n * 16 + i] = 0.f;
    __syncthreads();
    for (int p = threadIdx.x; p < n_pairs; p += blockDim.x) atomicAdd(&cursor_s[ch.expert(p)], 1);
    __syncthreads();
    if (wave == 0) {                                                         // where each expert's pairs begin, and the experts in use
        constexpr int PER = FEW_MAX_EXPERTS / WAVE;
        int count[PER], pairs = 0, used = 0;
#pragma unroll
        for (int i = 0; i < PER; ++i) {
            const int e = lane * PER + i;
            count[i] = e < experts ? cursor_s[e] : 0;
            pairs += count[i];
            used += count[i] > 0;
        }
        int pairs_to = pairs, used_to = used;                                // sums over the lanes up to this one
#pragma unroll
        for (int off = 1; off < WAVE; off <<= 1) {
            const int a = __shfl_up(pairs_to, off, WAVE), b = __shfl_up(used_to, off, WAVE);
            if (lane >= off) { pairs_to += a; used_to += b; }
        }
        int at = pairs_to - pairs, slot = used_to - used;
#pragma unroll
        for (int i = 0; i < PER; ++i) {
            const int e = lane * PER + i;
            if (e < experts) {
                start_s[e] = cursor_s[e] = at;
                if (count[i] > 0) used_s[slot++] = e;
            }
            at += count[i];
        }
        if (lane == WAVE - 1) { start_s[experts] = pairs_to; n_used_s = used_to; }
    }
    __syncthreads();
    for (int p = threadIdx.x; p < n_pairs; p += blockDim.x) sorted[atomicAdd(&cursor_s[ch.expert(p)], 1)] = p;
    __syncthreads();

    const int per_expert = (ff + FEW_PIECE - 1) / FEW_PIECE, of_experts = n_used_s * per_expert;
    const int items = of_experts + (shared_ff + FEW_PIECE - 1) / FEW_PIECE;
    float* mine = sums + wave * n * 16;
    for (int i = plane + planes * wave; i < items; i += planes * FEW_DOWN_WAVES) {
        const bool is_shared = i >= of_experts;
        const int e = is_shared ? 0 : used_s[i / per_expert];
        const int k0 = (is_shared ? i - of_experts : i % per_expert) * FEW_PIECE, my_ff = is_shared ? shared_ff : ff;
        const int k1 = min(my_ff, k0 + FEW_PIECE);
        const int first = is_shared ? 0 : start_s[e], m = is_shared ? n : start_s[e + 1] - first;
        const bf16_t* w_row = (is_shared ? shared_down : down + (size_t)e * width * ff) + (size_t)min(j0 + r, width - 1) * my_ff;
        for (int c0 = 0; c0 < m;) {
            const int left = m - c0;
#define FEW_DOWN(CT) { few_down_tile<CT>(mid, w_row, sorted + first, c0, m, is_shared, ch, ff, row_ff, k0, k1, r, g, mine); c0 += 16 * CT; }
            if (left > 32) FEW_DOWN(4) else if (left > 16) FEW_DOWN(2) else FEW_DOWN(1)
#undef FEW_DOWN
        }
    }
    __syncthreads();
    for (int i = threadIdx.x; i < n * 16; i += blockDim.x) {
        const int t = i / 16, j = j0 + i % 16;
        if (j >= width) continue;
        float total = 0.f;
#pragma unroll
        for (int w = 0; w < FEW_DOWN_WAVES; ++w) total += sums[w * n * 16 + i];
        if (plane == 0 && add0) total += to_float(add0[(size_t)t * width + j]);
        if (plane == 0 && add1) total += to_float(add1[(size_t)t * width + j]);
        out[((size_t)plane * n + t) * width + j] = total;
    }
}

// How many planes of partial sums fill the chip, for a reader that adds them (at most four).
PALM_API int palm_moe_few_planes(int width) {
    const int tiles = (width + 15) / 16;
    return tiles >= 512 ? 1 : min(4, (512 + tiles - 1) / tiles);
}

// h bfloat16 [n, width]; up, down, shared_up, shared_down, forms as in moe.hip, all bfloat16; chosen, weight [n, top], or with ids [n]
// the table [vocab, top] and no weight; add0, add1: null or bfloat16 rows [n, width]; mid: room for n * (top * ff + shared_ff) bfloat16;
// out float32 [planes, n, width].
PALM_API int palm_moe_few(hipStream_t stream, const void* h, const void* up, const void* down, const int* chosen, const float* weight,
                          const int* ids, int vocab, int n_tokens, int top, int experts, int width, int ff, const void* shared_up,
                          const void* shared_down, int shared_ff, int form, float limit, float slope, float shift, const void* add0,
                          const void* add1, void* mid, int planes, float* out) {
    PALM_CHECK(form >= EXPERT_GATED_SILU && form <= EXPERT_RELU_SQUARED, "moe_few: form %d is neither gated silu (0) nor plain gelu (1) nor capped "
               "gated (2) nor squared relu (3)", form);
    PALM_CHECK(form != EXPERT_CAPPED || limit > 0.f, "moe_few: the cap %g must be positive", (double)limit);
    PALM_CHECK(n_tokens >= 0 && n_tokens <= FEW_ROWS && top > 0 && top <= experts && experts <= FEW_MAX_EXPERTS && width > 0 && ff > 0,
               "moe_few: n=%d (at most %d) top=%d experts=%d (at most %d) width=%d ff=%d", n_tokens, FEW_ROWS, top, experts, FEW_MAX_EXPERTS, width, ff);
    PALM_CHECK(n_tokens * top <= FEW_MAX_PAIRS, "moe_few: %d rows x %d choices exceed %d", n_tokens, top, FEW_MAX_PAIRS);
    PALM_CHECK(width % 8 == 0 && ff % 8 == 0 && shared_ff % 8 == 0 && shared_ff >= 0, "moe_few: width %d and inner sizes %d, %d must be multiples of "
               "eight", width, ff, shared_ff);
    PALM_CHECK(ids ? vocab > 0 : weight != nullptr, "moe_few: choices come with weights, or from a table of %d ids", vocab);
    PALM_CHECK(shared_ff == 0 || (shared_up && shared_down), "moe_few: a shared expert of inner size %d needs its matrices", shared_ff);
    PALM_CHECK(planes >= 1 && planes <= 4, "moe_few: %d planes (at most four)", planes);
    if (n_tokens == 0) return 0;
    const FewChoices ch{chosen, weight, ids, vocab, top, n_tokens};
    const ExpertCap cap{limit, slope, shift};
    const int longest = max(ff, shared_ff), runs = (longest + 16 * FEW_UP_WAVES - 1) / (16 * FEW_UP_WAVES);
    PALM_CHECK(runs <= 65535, "moe_few: an inner size of %d is more than one launch takes", longest);
    const dim3 grid(experts + (shared_ff > 0), runs);
#define FEW_LAUNCH(GATED) moe_few_up_kernel<GATED><<<grid, 2 * FEW_UP_WAVES * WAVE, 0, stream>>>((const bf16_t*)h, (const bf16_t*)up, ch, experts, width, ff, \
        (const bf16_t*)shared_up, shared_ff, form, cap, (bf16_t*)mid)
    if (expert_is_gated(form)) FEW_LAUNCH(true); else FEW_LAUNCH(false);
#undef FEW_LAUNCH
    const size_t lds = (size_t)FEW_DOWN_WAVES * n_tokens * 16 * sizeof(float) + (size_t)n_tokens * top * sizeof(int);
    moe_few_down_kernel<<<dim3((width + 15) / 16, planes), FEW_DOWN_WAVES * WAVE, lds, stream>>>(
        (const bf16_t*)mid, (const bf16_t*)down, ch, experts, width, ff, (const bf16_t*)shared_down, shared_ff, (const bf16_t*)add0,
        (const bf16_t*)add1, out);
    PALM_LAUNCHED();
    return 0;
}
