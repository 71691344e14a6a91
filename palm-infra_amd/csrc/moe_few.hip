// Routed experts for few rows (a decode step's batch) in bfloat16 on the matrix cores.  Every expert that somebody chose has its
// matrices read once, whatever the number of rows that chose it; nothing is planned on the host and no launch of its own plans.
//
//   up     a block per (expert, run of matrix rows): the block finds the rows that chose its expert (none: it is done) and
//          brings their activations into LDS, and each wave streams 16 rows of the expert's first matrix (gated forms: 16 gate
//          rows and their 16 up rows) past them, 16 rows of activations a column tile; mid[t, c, f] = act(..) in bfloat16, t's choices one after the other, the shared
//          expert's values behind them
//   down   a block per (16 output features, plane): all (row, choice) pairs are sorted by expert in LDS; pieces of 256 inner
//          values of the experts in use are dealt to the planes' waves in turn; a piece's products go, weighted, into the wave's
//          own sums [row, 16 features] in LDS, and the waves' sums are added in their order
//
// Both kernels are made for up to 16 rows (one column tile) and for more (up to four that share every matrix fragment).
//
// A shared expert that every row goes through (weight one, an inner size of its own) runs as one more expert.  Result: float32
// planes [planes, n, width] for a reader that adds them, the first with the rows of other branches.
#include "mfma.h"
#include "expert_form.h"

constexpr int FEW_ROWS = 128;                     // rows of a step at most
constexpr int FEW_UP_WAVES = 4;
constexpr int FEW_DOWN_WAVES = 8;
constexpr int FEW_STEPS = 8;                      // reads of 32 values of every matrix row under way together
constexpr int FEW_PIECE = 32 * FEW_STEPS;         // inner values of a piece
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

// acc[ct] += (16 matrix rows) x (16 rows of activations in column tile ct) over one piece k0 .. k1: lane (r, g) reads row r of each, the
// eight values of group g of every step of 32.  w_row: this lane's matrix row; xr: its activation rows.
template <int CT>
__device__ inline void few_piece(const bf16_t* w_row, const bf16_t* const (&xr)[CT], int k0, int k1, int g, f32x4 (&acc)[CT]) {
    bf16x8 wf[FEW_STEPS];
#pragma unroll
    for (int s = 0; s < FEW_STEPS; ++s) wf[s] = few_row8(w_row, k0 + 32 * s + 8 * g, k1);
#pragma unroll
    for (int s = 0; s < FEW_STEPS; ++s)
#pragma unroll
        for (int ct = 0; ct < CT; ++ct) acc[ct] = mfma_16x16x32(wf[s], few_row8(xr[ct], k0 + 32 * s + 8 * g, k1), acc[ct]);
}

// Activations for the first products: the columns' rows in LDS, a segment of the inner size at a time.
// (The matrices come in order through one counter of loads: activations read from memory between them would make every wait for
// them a wait for the rows asked for ahead.)
constexpr int few_segment(int max_ct) { return max_ct == 1 ? 2048 : 512; }
constexpr int FEW_PAD = 8;                         // elements between a segment's end and the next row: rows begin in different banks

template <bool GATED, int MAX_CT>
__global__ __launch_bounds__(FEW_UP_WAVES * WAVE) void moe_few_up_kernel(const bf16_t* __restrict__ h, const bf16_t* __restrict__ up, FewChoices ch,
                                                                         int experts, int width, int ff, const bf16_t* __restrict__ shared_up,
                                                                         int shared_ff, int form, ExpertCap cap, bf16_t* __restrict__ mid) {
    constexpr int MATS = GATED ? 2 : 1, COLS = 16 * MAX_CT;
    extern __shared__ __attribute__((aligned(16))) bf16_t x_s[];     // [columns][segment + FEW_PAD]
    __shared__ int list_s[FEW_MAX_PAIRS];
    __shared__ int count_s;
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
    if (m == 0) return;
    const int lane = threadIdx.x % WAVE, wave = threadIdx.x / WAVE;
    const int r = lane % 16, g = lane / 16, f0 = block_f + 16 * wave;   // (rows beyond the matrix: its last one again, not kept)
    const bf16_t* w = is_shared ? shared_up : up + (size_t)e * MATS * ff * width;
    const bf16_t* wr[MATS];
    wr[0] = w + (size_t)min(f0 + r, my_ff - 1) * width;
    if constexpr (GATED) wr[1] = wr[0] + (size_t)my_ff * width;
    const int segment = min(width, few_segment(MAX_CT)), stride = segment + FEW_PAD;
    for (int c0 = 0; c0 < m; c0 += COLS) {
        const int cols = min(COLS, m - c0);
        f32x4 acc[MATS][MAX_CT];
#pragma unroll
        for (int i = 0; i < MATS; ++i)
#pragma unroll
            for (int ct = 0; ct < MAX_CT; ++ct) acc[i][ct] = f32x4{0.f, 0.f, 0.f, 0.f};
        for (int k0 = 0; k0 < width; k0 += segment) {
            const int k1 = min(width, k0 + segment), len = k1 - k0;
            // the first chunk's matrix rows are on their way while the activations go to LDS
            constexpr int CHUNK = 32 * FEW_STEPS;
            bf16x8 wf[MATS][FEW_STEPS];
            auto read = [&](int k, bf16x8 (&to)[MATS][FEW_STEPS]) {
#pragma unroll
                for (int i = 0; i < MATS; ++i)
#pragma unroll
                    for (int s = 0; s < FEW_STEPS; ++s) to[i][s] = load_bf16x8(wr[i] + min(k + 32 * s + 8 * g, k1 - 8));   // (beyond the end: met by zeros)
            };
            read(k0, wf);
            __syncthreads();                                         // (whoever still reads the segment before is done)
            for (int i = threadIdx.x; i < cols * (len / 8); i += blockDim.x) {
                const int col = i / (len / 8), d = i % (len / 8) * 8;
                const int p = list_s[c0 + col];
                *reinterpret_cast<uint4*>(x_s + (size_t)col * stride + d) = *reinterpret_cast<const uint4*>(h + (size_t)(is_shared ? p : p / ch.top) * width + k0 + d);
            }
            __syncthreads();
            for (int k = k0; k < k1; k += CHUNK) {
                bf16x8 next[MATS][FEW_STEPS];
                read(min(k + CHUNK, k1 - 8), next);                  // (after the last chunk: its end once more, not used)
#pragma unroll
                for (int s = 0; s < FEW_STEPS; ++s) {
                    const int d = k - k0 + 32 * s + 8 * g;
#pragma unroll
                    for (int ct = 0; ct < MAX_CT; ++ct) {
                        if (16 * ct >= cols) continue;               // (the same in every lane)
                        bf16x8 x = *reinterpret_cast<const bf16x8*>(x_s + (size_t)min(16 * ct + r, cols - 1) * stride + min(d, len - 8));
                        if (d >= len) x = zero_bf16x8();
#pragma unroll
                        for (int i = 0; i < MATS; ++i) acc[i][ct] = mfma_16x16x32(wf[i][s], x, acc[i][ct]);
                    }
                }
#pragma unroll
                for (int i = 0; i < MATS; ++i)
#pragma unroll
                    for (int s = 0; s < FEW_STEPS; ++s) wf[i][s] = next[i][s];
            }
        }
        // lane (r, g) holds inner values f0 + 4 g + i of column r
#pragma unroll
        for (int ct = 0; ct < MAX_CT; ++ct) {
            const int col = 16 * ct + r, f = f0 + 4 * g;
            if (col >= cols || f >= my_ff) continue;
            const int p = list_s[c0 + col];
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
    f32x4 acc[CT];
#pragma unroll
    for (int ct = 0; ct < CT; ++ct) acc[ct] = f32x4{0.f, 0.f, 0.f, 0.f};
    few_piece<CT>(w_row, xr, k0, k1, g, acc);
    // lane (r, g) holds features 4 g + i of column r; the columns of a tile are different rows
#pragma unroll
    for (int ct = 0; ct < CT; ++ct) {
        if (c0 + 16 * ct + r >= m) continue;
        float4* to = reinterpret_cast<float4*>(sums + token[ct] * 16 + 4 * g);
        float4 v = *to;
        v.x = fmaf(weight[ct], acc[ct][0], v.x); v.y = fmaf(weight[ct], acc[ct][1], v.y);
        v.z = fmaf(weight[ct], acc[ct][2], v.z); v.w = fmaf(weight[ct], acc[ct][3], v.w);
        *to = v;
    }
}

template <int MAX_CT>
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
            if constexpr (MAX_CT == 1) FEW_DOWN(1) else if (left > 32) FEW_DOWN(4) else if (left > 16) FEW_DOWN(2) else FEW_DOWN(1)
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
#define FEW_LAUNCH(GATED, MAX_CT) moe_few_up_kernel<GATED, MAX_CT><<<grid, FEW_UP_WAVES * WAVE, \
        (size_t)min(n_tokens, 16 * MAX_CT) * (min(width, few_segment(MAX_CT)) + FEW_PAD) * sizeof(bf16_t), stream>>>( \
        (const bf16_t*)h, (const bf16_t*)up, ch, experts, width, ff, (const bf16_t*)shared_up, shared_ff, form, cap, (bf16_t*)mid)
    if (n_tokens <= 16) {
        if (expert_is_gated(form)) FEW_LAUNCH(true, 1); else FEW_LAUNCH(false, 1);
    } else {
        if (expert_is_gated(form)) FEW_LAUNCH(true, 4); else FEW_LAUNCH(false, 4);
    }
#undef FEW_LAUNCH
    const size_t lds = (size_t)FEW_DOWN_WAVES * n_tokens * 16 * sizeof(float) + (size_t)n_tokens * top * sizeof(int);
#define FEW_LAUNCH(MAX_CT) moe_few_down_kernel<MAX_CT><<<dim3((width + 15) / 16, planes), FEW_DOWN_WAVES * WAVE, lds, stream>>>( \
        (const bf16_t*)mid, (const bf16_t*)down, ch, experts, width, ff, (const bf16_t*)shared_down, shared_ff, (const bf16_t*)add0, \
        (const bf16_t*)add1, out)
    if (n_tokens <= 16) FEW_LAUNCH(1); else FEW_LAUNCH(4);
#undef FEW_LAUNCH
    PALM_LAUNCHED();
    return 0;
}
