// Routed experts for many rows (a prompt), planned on the device: the (token, choice) pairs are grouped by expert, and two
// grouped products on the matrix cores run all experts' rows in one launch each.
//
//   plan      count the pairs of every expert; pad every expert's run of pairs to whole tiles of rows and lay the
//             runs one after the other; place every pair in its run, in no particular order (a slot is a column of the
//             products by itself: no result depends on where in its run a pair lies); the slots that pad a run hold -1
//   grouped   for every tile (its expert comes from the plan): mid = silu(G_e x) * (U_e x) for the tile's rows x, then
//             y = D_e mid.  The weights are the first operand of the matrix instruction, so that a lane ends with four
//             neighbouring features of one row.  Sizes in whole cache lines with enough rows an expert: blocks of 128 rows x 256
//             features through a ring of stages in LDS (moe_tile_kernel).  Otherwise a wave owns 32 features x 64 rows and reads its
//             fragments from memory itself (a weight fragment feeds four products, a row fragment two or four)
//   combine   out[t] = sum_c weight[t, c] * y[place of pair (t, c)], in the order of c, 32-bit, plus up to two rows that other
//             branches made
#include "mfma.h"
#include "expert_form.h"
#include "lds_stage.h"

constexpr int GT_TOKENS = 64;                     // rows of a tile whose fragments come from memory
constexpr int GT_RUNS = GT_TOKENS / 16;           // runs of 16 rows: what one matrix instruction takes
constexpr int GT_WAVES = 4;
constexpr int GT_FEATURES = 32 * GT_WAVES;        // features of a block's tile
constexpr int PLAN_THREADS = 1024;
constexpr int PLAN_MAX_EXPERTS = 512;

__device__ inline bf16x8 grouped_row8(const bf16_t* row, int col, int dim) {
    // eight values of a row from column `col`; columns beyond `dim` are zero (dim is a multiple of eight); the read itself
    // is unconditional
    const bf16x8 v = load_bf16x8(row + min(col, dim - 8));
    return col < dim ? v : zero_bf16x8();
}

// One block.  starts[e] = first slot of expert e's run (runs padded to whole tiles); tile_expert[i] = the expert of tile i, -1 beyond
// the last tile; slot_pair[slot] = pair (-1 where a run is padded), pair_slot[pair] = slot.  The choices are rows [n, top], or with
// ids the rows of a table [vocab, top] that the tokens' ids pick.
__global__ __launch_bounds__(PLAN_THREADS) void moe_plan_kernel(const int* __restrict__ chosen, const int* __restrict__ ids, int vocab, int top,
                                                                int n_pairs, int experts, int max_tiles, int tile,
                                                                int* __restrict__ tile_expert, int* __restrict__ slot_pair,
                                                                int* __restrict__ pair_slot) {
    __shared__ int start_s[PLAN_MAX_EXPERTS + 1], cursor_s[PLAN_MAX_EXPERTS];
    const int lane = threadIdx.x % WAVE;
    auto choice = [&](int p) { return ids ? chosen[(size_t)min(max(ids[p / top], 0), vocab - 1) * top + p % top] : chosen[p]; };
    for (int e = threadIdx.x; e < experts; e += PLAN_THREADS) cursor_s[e] = 0;
    __syncthreads();
    for (int p = threadIdx.x; p < n_pairs; p += PLAN_THREADS) atomicAdd(&cursor_s[choice(p)], 1);
    __syncthreads();
    if (threadIdx.x < WAVE) {
        constexpr int PER = PLAN_MAX_EXPERTS / WAVE;
        int padded[PER], mine = 0;
#pragma unroll
        for (int i = 0; i < PER; ++i) {
            const int e = lane * PER + i;
            padded[i] = e < experts ? (cursor_s[e] + tile - 1) / tile * tile : 0;
            mine += padded[i];
        }
        int up_to = mine;                                             // the sum over the lanes up to this one
#pragma unroll
        for (int off = 1; off < WAVE; off <<= 1) {
            const int other = __shfl_up(up_to, off, WAVE);
            if (lane >= off) up_to += other;
        }
        int at = up_to - mine;
#pragma unroll
        for (int i = 0; i < PER; ++i) {
            const int e = lane * PER + i;
            if (e < experts) start_s[e] = at;
            at += padded[i];
        }
        if (lane == WAVE - 1) start_s[experts] = up_to;
    }
    __syncthreads();
    for (int i = threadIdx.x; i < max_tiles; i += PLAN_THREADS) tile_expert[i] = -1;
    // the slots that pad each run
    for (int e = threadIdx.x / WAVE; e < experts; e += PLAN_THREADS / WAVE)
        for (int s = start_s[e] + cursor_s[e] + lane; s < start_s[e + 1]; s += WAVE) slot_pair[s] = -1;
    __syncthreads();
    for (int e = threadIdx.x; e < experts; e += PLAN_THREADS) {
        for (int i = start_s[e] / tile; i < start_s[e + 1] / tile; ++i) tile_expert[i] = e;
        cursor_s[e] = start_s[e];
    }
    __syncthreads();
    for (int p = threadIdx.x; p < n_pairs; p += PLAN_THREADS) {
        const int slot = atomicAdd(&cursor_s[choice(p)], 1);
        slot_pair[slot] = p;
        pair_slot[p] = slot;
    }
}

// grid (tiles, blocks of GT_FEATURES features).  a: the rows [*, k_dim]; row_of_slot: null (the rows lie in slot order) or
// slot -> pair, the pair's row being pair / top.  w: [experts, n_w_rows, k_dim]; FORM 1 (gated): n_w_rows = 2 n_features, an
// expert's gate rows first, and the result is silu(gate) * up; FORM 3: the same rows, capped gated; FORM 2: the product through
// the exact gelu; FORM 4: the product through the squared relu; FORM 0: the product as it is.  out: bfloat16 [slots, n_features].
template <int FORM>
__global__ __launch_bounds__(GT_WAVES * WAVE) void moe_grouped_kernel(const bf16_t* __restrict__ a, const int* __restrict__ slot_pair, int top,
                                                                      const bf16_t* __restrict__ w, const int* __restrict__ tile_expert,
                                                                      int n_features, int k_dim, ExpertCap cap, bf16_t* __restrict__ out) {
    constexpr bool GATED = FORM == 1 || FORM == 3;
    const int tile = blockIdx.x;
    const int e = tile_expert[tile];
    if (e < 0) return;
    const int lane = threadIdx.x % WAVE, wave = threadIdx.x / WAVE;
    const int r = lane % 16, g = lane / 16;
    const int f0 = blockIdx.y * GT_FEATURES + wave * 32;
    if (f0 >= n_features) return;
    const int slot0 = tile * GT_TOKENS;
    // the rows of the tile's runs of 16 slots, as the second operand: column r is a row of activations
    const bf16_t* ar[GT_RUNS];
#pragma unroll
    for (int tt = 0; tt < GT_RUNS; ++tt) {
        const int slot = slot0 + 16 * tt + r;
        const int pair = slot_pair ? slot_pair[slot] : slot;
        const int row = slot_pair ? max(pair, 0) / top : slot;          // a slot that pads the run reads row 0; nobody reads its result
        ar[tt] = a + (size_t)row * k_dim;
    }
    const size_t w_rows = GATED ? 2 * (size_t)n_features : (size_t)n_features;
    const bf16_t* wr[GATED ? 4 : 2];
#pragma unroll
    for (int ft = 0; ft < 2; ++ft) {
        const int f = min(f0 + 16 * ft + r, n_features - 1);
        wr[ft] = w + ((size_t)e * w_rows + f) * k_dim;
        if (GATED) wr[2 + ft] = w + ((size_t)e * w_rows + n_features + f) * k_dim;
    }
    f32x4 acc[GATED ? 4 : 2][GT_RUNS];
#pragma unroll
    for (int i = 0; i < (GATED ? 4 : 2); ++i)
#pragma unroll
        for (int tt = 0; tt < GT_RUNS; ++tt) acc[i][tt] = f32x4{0.f, 0.f, 0.f, 0.f};
    for (int k0 = 0; k0 < k_dim; k0 += 32) {
        const int col = k0 + 8 * g;
        bf16x8 af[GT_RUNS], wf[GATED ? 4 : 2];
#pragma unroll
        for (int tt = 0; tt < GT_RUNS; ++tt) af[tt] = grouped_row8(ar[tt], col, k_dim);
#pragma unroll
        for (int i = 0; i < (GATED ? 4 : 2); ++i) wf[i] = grouped_row8(wr[i], col, k_dim);
#pragma unroll
        for (int i = 0; i < (GATED ? 4 : 2); ++i)
#pragma unroll
            for (int tt = 0; tt < GT_RUNS; ++tt) acc[i][tt] = mfma_16x16x32(wf[i], af[tt], acc[i][tt]);
    }
    // lane (r, g) holds features f0 + 16 ft + 4 g + i of the row in slot slot0 + 16 tt + r
#pragma unroll
    for (int ft = 0; ft < 2; ++ft)
#pragma unroll
        for (int tt = 0; tt < GT_RUNS; ++tt) {
            const int f = f0 + 16 * ft + 4 * g;
            if (f >= n_features) continue;                              // n_features is a multiple of four
            float v[4];
#pragma unroll
            for (int i = 0; i < 4; ++i) {
                if (GATED) {
                    v[i] = FORM == 3 ? expert_capped(acc[ft][tt][i], acc[2 + ft][tt][i], cap) : expert_silu_gated(acc[ft][tt][i], acc[2 + ft][tt][i]);
                } else if (FORM == 2) {
                    v[i] = expert_gelu(acc[ft][tt][i]);
                } else if (FORM == 4) {
                    v[i] = expert_relu_squared(acc[ft][tt][i]);
                } else {
                    v[i] = acc[ft][tt][i];
                }
            }
            uint2 pk;
            pk.x = (uint32_t)f32_to_bf16(v[0]).bits | ((uint32_t)f32_to_bf16(v[1]).bits << 16);
            pk.y = (uint32_t)f32_to_bf16(v[2]).bits | ((uint32_t)f32_to_bf16(v[3]).bits << 16);
            *reinterpret_cast<uint2*>(out + (size_t)(slot0 + 16 * tt + r) * n_features + f) = pk;
        }
}

// The same products with both operands crossing LDS.  A block of eight waves owns TILE_ROWS slots x TILE_W_ROWS rows of an
// expert's matrix and walks over K in stages of 64 (a row of a stage is one cache line of 128 bytes), the stages in a ring
// that global_load_lds fills; a row's eight 16-byte chunks are permuted by the row's number so that an operand's reads spread
// over the banks (the lane that fills a place fetches the chunk that belongs there).  MFMA 32x32x16: 32 weight rows x 32 slots, a wave
// owns 64 weight rows x 64 slots.  Gated forms: of every 64 weight rows of a tile the first 32 are gate rows and the others
// their up rows.  FORM as above.  The tiles of an expert that lies in the plan follow each other, features innermost, and each
// die gets a run of neighbouring tiles.
typedef float f32x16 __attribute__((ext_vector_type(16)));
constexpr int TILE_ROWS = 128, TILE_W_ROWS = 256, TILE_K = 64, TILE_WAVES = 8, TILE_WAVES_F = 4;
constexpr int TILE_LINE = TILE_K * 2, TILE_CHUNKS = TILE_LINE / 16, TILE_RING = 3;
constexpr int TILE_STAGE = (TILE_ROWS + TILE_W_ROWS) * TILE_LINE;
constexpr int TILE_LOADS = TILE_STAGE / 1024 / TILE_WAVES;            // instructions a wave and stage
constexpr int TILE_DIES = 8;

template <int FORM>
__global__ __launch_bounds__(TILE_WAVES * WAVE) void moe_tile_kernel(const bf16_t* __restrict__ a, const int* __restrict__ slot_pair, int top,
                                                                     const bf16_t* __restrict__ w, const int* __restrict__ tile_expert,
                                                                     int max_tiles, int feature_tiles, int n_features, int k_dim,
                                                                     ExpertCap cap, bf16_t* __restrict__ out) {
    constexpr bool GATED = FORM == 1 || FORM == 3;
    constexpr int TILE_FEATURES = GATED ? TILE_W_ROWS / 2 : TILE_W_ROWS;
    __shared__ __attribute__((aligned(1024))) char lds[TILE_RING * TILE_STAGE];
    const int total = max_tiles * feature_tiles, per_die = (total + TILE_DIES - 1) / TILE_DIES;
    const int pid = (blockIdx.x % TILE_DIES) * per_die + blockIdx.x / TILE_DIES;
    if (pid >= total) return;
    const int tile = pid / feature_tiles, f0 = pid % feature_tiles * TILE_FEATURES;
    const int e = tile_expert[tile];
    if (e < 0) return;
    const int lane = threadIdx.x % WAVE, wave = __builtin_amdgcn_readfirstlane(threadIdx.x / WAVE);
    const int wave_f = wave % TILE_WAVES_F, wave_t = wave / TILE_WAVES_F;
    const bf16_t* we = w + (size_t)e * (GATED ? 2 : 1) * n_features * k_dim;

    // the rows this lane brings in: instruction q of this wave fills the stage's rows (q * 8 + wave) * 8 .. + 7, weights first
    const char* src[TILE_LOADS];
#pragma unroll
    for (int q = 0; q < TILE_LOADS; ++q) {
        const int R = (q * TILE_WAVES + wave) * 8 + lane / TILE_CHUNKS;
        const int chunk = (lane % TILE_CHUNKS) ^ ((R >> 1) & (TILE_CHUNKS - 1));
        const bf16_t* row;
        if (R < TILE_W_ROWS) {
            const int f = GATED ? f0 + R / 64 * 32 + R % 32 : f0 + R;
            row = we + ((size_t)min(f, n_features - 1) + (GATED && R / 32 % 2 ? n_features : 0)) * k_dim;
        } else {
            const int slot = tile * TILE_ROWS + R - TILE_W_ROWS;
            // a slot that pads the run reads row 0; nobody reads its result
            row = a + (size_t)(slot_pair ? max(slot_pair[slot], 0) / top : slot) * k_dim;
        }
        src[q] = reinterpret_cast<const char*>(row) + chunk * 16;
    }
    const uint32_t lds0 = __builtin_amdgcn_readfirstlane((uint32_t)(uintptr_t)(__attribute__((address_space(3))) const void*)lds);
    auto bring = [&](int kt, int place) {
#pragma unroll
        for (int q = 0; q < TILE_LOADS; ++q)
            row_chunk_into_lds(src[q] + (size_t)kt * TILE_LINE, lds0 + place * TILE_STAGE + (q * TILE_WAVES + wave) * 1024);
    };
    int w_off[2], x_off[2], cs[TILE_K / 16];
#pragma unroll
    for (int i = 0; i < 2; ++i) {
        w_off[i] = (wave_f * 64 + i * 32 + lane % 32) * TILE_LINE;
        x_off[i] = (TILE_W_ROWS + wave_t * 64 + i * 32 + lane % 32) * TILE_LINE;
    }
#pragma unroll
    for (int s = 0; s < TILE_K / 16; ++s) cs[s] = ((2 * s + lane / 32) ^ ((lane >> 1) & (TILE_CHUNKS - 1))) * 16;
    f32x16 acc[2][2];
#pragma unroll
    for (int f = 0; f < 2; ++f)
#pragma unroll
        for (int t = 0; t < 2; ++t)
#pragma unroll
            for (int v = 0; v < 16; ++v) acc[f][t][v] = 0.f;

    const int stages = k_dim / TILE_K;
    constexpr int AHEAD = TILE_RING - 1;
#pragma unroll
    for (int i = 0; i < AHEAD; ++i)
        if (i < stages) bring(i, i);
    int place = 0;
    for (int kt = 0; kt < stages; ++kt) {
        if (kt + AHEAD <= stages) all_but_the_youngest_have_arrived<(AHEAD - 1) * TILE_LOADS>();
        else all_but_the_youngest_have_arrived<0>();
        __syncthreads();                                       // every wave's share of the stage; and everyone is done with the one before
        if (kt + AHEAD < stages) bring(kt + AHEAD, place == 0 ? TILE_RING - 1 : place - 1);
        const char* stage = lds + place * TILE_STAGE;
        bf16x8 wf[2][2], xf[2][2];
        auto read_operands = [&](int s) {
#pragma unroll
            for (int i = 0; i < 2; ++i) {
                wf[s & 1][i] = *reinterpret_cast<const bf16x8*>(stage + w_off[i] + cs[s]);
                xf[s & 1][i] = *reinterpret_cast<const bf16x8*>(stage + x_off[i] + cs[s]);
            }
        };
        read_operands(0);
#pragma unroll
        for (int s = 0; s < TILE_K / 16; ++s) {
            if (s + 1 < TILE_K / 16) read_operands(s + 1);
#pragma unroll
            for (int f = 0; f < 2; ++f)
#pragma unroll
                for (int t = 0; t < 2; ++t)
                    acc[f][t] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(wf[s & 1][f], xf[s & 1][t], acc[f][t], 0, 0, 0);
            if (s + 1 < TILE_K / 16) {
#pragma unroll
                for (int i = 0; i < 4; ++i) {
                    __builtin_amdgcn_sched_group_barrier(0x008, 1, 0);      // one matrix instruction
                    __builtin_amdgcn_sched_group_barrier(0x100, 1, 0);      // one LDS read
                }
            }
        }
        place = place + 1 == TILE_RING ? 0 : place + 1;
    }

    // element v of a result tile: slot lane % 32, weight row 8 (v / 4) + 4 (lane / 32) + v % 4
#pragma unroll
    for (int t = 0; t < 2; ++t) {
        const size_t slot = (size_t)tile * TILE_ROWS + wave_t * 64 + t * 32 + lane % 32;
#pragma unroll
        for (int f = 0; f < (GATED ? 1 : 2); ++f)
#pragma unroll
            for (int q4 = 0; q4 < 4; ++q4) {
                const int feat = f0 + (GATED ? wave_f * 32 : wave_f * 64 + f * 32) + 8 * q4 + 4 * (lane / 32);
                if (feat >= n_features) continue;              // n_features is a multiple of four
                bf16_t v[4];
#pragma unroll
                for (int i = 0; i < 4; ++i) {
                    const float z = acc[f][t][4 * q4 + i];
                    v[i] = f32_to_bf16(FORM == 1 ? expert_silu_gated(z, acc[1][t][4 * q4 + i]) : FORM == 3 ? expert_capped(z, acc[1][t][4 * q4 + i], cap)
                                       : FORM == 2 ? expert_gelu(z) : FORM == 4 ? expert_relu_squared(z) : z);
                }
                *reinterpret_cast<uint2*>(out + slot * n_features + feat) = make_uint2((uint32_t)v[0].bits | ((uint32_t)v[1].bits << 16),
                                                                                       (uint32_t)v[2].bits | ((uint32_t)v[3].bits << 16));
            }
    }
}

// One block per token; eight neighbouring columns a thread (width is a multiple of eight).  weight: null, or [n, top] (null: 1 / top).
__global__ void moe_combine_kernel(const bf16_t* __restrict__ y, const int* __restrict__ pair_slot, const float* __restrict__ weight, int top,
                                   int width, const bf16_t* __restrict__ add0, const bf16_t* __restrict__ add1, float* __restrict__ out) {
    const size_t t = blockIdx.x;
    for (int d = threadIdx.x * 8; d < width; d += blockDim.x * 8) {
        float total[8];
#pragma unroll
        for (int i = 0; i < 8; ++i) total[i] = 0.f;
        auto add = [&](const bf16_t* row, float f) {
            const bf16x8 v = load_bf16x8(row + d);
#pragma unroll
            for (int i = 0; i < 8; ++i) total[i] = fmaf(f, (float)v[i], total[i]);
        };
#pragma unroll 4
        for (int c = 0; c < top; ++c)
            add(y + (size_t)pair_slot[t * top + c] * width, weight ? weight[t * top + c] : 1.0f / (float)top);
        if (add0) add(add0 + t * width, 1.0f);
        if (add1) add(add1 + t * width, 1.0f);
        *reinterpret_cast<float4*>(out + t * width + d) = make_float4(total[0], total[1], total[2], total[3]);
        *reinterpret_cast<float4*>(out + t * width + d + 4) = make_float4(total[4], total[5], total[6], total[7]);
    }
}

// Rows of a tile: the kernel whose operands cross LDS takes sizes in whole lines and pays from some 40 rows an expert on.
static int tile_of(long long n_pairs, int experts, int width, int ff) {
    return width % TILE_K == 0 && ff % TILE_K == 0 && n_pairs >= 40ll * experts ? TILE_ROWS : GT_TOKENS;
}
PALM_API int palm_moe_tile_tokens(int n_pairs, int experts, int width, int ff) { return tile_of(n_pairs, experts, width, ff); }

// chosen, weight [n, top]; h bfloat16 [n, width]; gate_up bfloat16 [experts, 2 ff, width] (the plain forms: [experts, ff, width], up
// rows alone); add0, add1: null or bfloat16 rows [n, width]; down bfloat16 [experts, width, ff].
// With ids [n] chosen is a table [vocab, top] of which every token takes its id's row, and weight may be null (1 / top).
// Room, with tile = palm_moe_tile_tokens(n top, experts, width, ff), max_tiles = ceil(n top / tile) + experts and slots = max_tiles * tile: plan: (max_tiles + slots
// + n top) ints; mid: slots * ff bfloat16; y: slots * width bfloat16.  out float32 [n, width].
PALM_API int palm_moe_grouped(hipStream_t stream, const void* h, const void* gate_up, const void* down, const int* chosen,
                              const float* weight, int n_tokens, int top, int experts, int width, int ff, int* plan, void* mid, void* y,
                              float* out, int form, float limit, float slope, float shift, const void* add0, const void* add1,
                              const int* ids, int vocab) {
    PALM_CHECK(ids ? vocab > 0 : weight != nullptr, "moe_grouped: choices come with weights, or from a table of %d ids", vocab);
    PALM_CHECK(experts <= PLAN_MAX_EXPERTS, "moe_grouped: %d experts exceed %d", experts, PLAN_MAX_EXPERTS);
    PALM_CHECK(form >= EXPERT_GATED_SILU && form <= EXPERT_RELU_SQUARED, "moe_grouped: form %d is neither gated silu (0) nor plain gelu (1) nor capped "
               "gated (2) nor squared relu (3)", form);
    PALM_CHECK(form != EXPERT_CAPPED || limit > 0.f, "moe_grouped: the cap %g must be positive", (double)limit);
    PALM_CHECK(n_tokens >= 0 && top > 0 && experts > 0 && width > 0 && ff > 0, "moe_grouped: n=%d top=%d experts=%d width=%d ff=%d", n_tokens,
               top, experts, width, ff);
    PALM_CHECK(width % 8 == 0 && ff % 8 == 0, "moe_grouped: width %d and inner size %d must be multiples of eight", width, ff);
    if (n_tokens == 0) return 0;
    const long long n_pairs = (long long)n_tokens * top;
    PALM_CHECK(n_pairs < (1ll << 30), "moe_grouped: %lld pairs are more than one launch takes", n_pairs);
    const int tile = tile_of(n_pairs, experts, width, ff);
    const int max_tiles = (int)((n_pairs + tile - 1) / tile) + experts;
    int* tile_expert = plan;
    int* slot_pair = tile_expert + max_tiles;
    int* pair_slot = slot_pair + (size_t)max_tiles * tile;
    moe_plan_kernel<<<1, PLAN_THREADS, 0, stream>>>(chosen, ids, vocab, top, (int)n_pairs, experts, max_tiles, tile, tile_expert, slot_pair, pair_slot);
    const int combine_threads = width >= 2048 ? 256 : 128;
    const ExpertCap cap{limit, slope, shift};
    if (tile == TILE_ROWS) {
        auto blocks = [&](int feature_tiles) { return dim3((max_tiles * feature_tiles + TILE_DIES - 1) / TILE_DIES * TILE_DIES); };
        const int up_features = expert_is_gated(form) ? TILE_W_ROWS / 2 : TILE_W_ROWS;
        const int up_tiles = (ff + up_features - 1) / up_features, down_tiles = (width + TILE_W_ROWS - 1) / TILE_W_ROWS;
        PALM_CHECK((long long)max_tiles * max(up_tiles, down_tiles) < (1ll << 30), "moe_grouped: %d tiles of rows are more than one launch takes", max_tiles);
#define MOE_TILE_UP(FORM) moe_tile_kernel<FORM><<<blocks(up_tiles), TILE_WAVES * WAVE, 0, stream>>>((const bf16_t*)h, slot_pair, top, \
            (const bf16_t*)gate_up, tile_expert, max_tiles, up_tiles, ff, width, cap, (bf16_t*)mid)
        if (form == EXPERT_GATED_SILU) MOE_TILE_UP(1);
        else if (form == EXPERT_GELU) MOE_TILE_UP(2);
        else if (form == EXPERT_CAPPED) MOE_TILE_UP(3);
        else MOE_TILE_UP(4);
#undef MOE_TILE_UP
        moe_tile_kernel<0><<<blocks(down_tiles), TILE_WAVES * WAVE, 0, stream>>>((const bf16_t*)mid, nullptr, top, (const bf16_t*)down, tile_expert,
                                                                                 max_tiles, down_tiles, width, ff, cap, (bf16_t*)y);
        moe_combine_kernel<<<n_tokens, combine_threads, 0, stream>>>((const bf16_t*)y, pair_slot, weight, top, width, (const bf16_t*)add0, (const bf16_t*)add1, out);
        PALM_LAUNCHED();
        return 0;
    }
    const dim3 up_grid(max_tiles, (ff + GT_FEATURES - 1) / GT_FEATURES);
#define MOE_UP(FORM) moe_grouped_kernel<FORM><<<up_grid, GT_WAVES * WAVE, 0, stream>>>((const bf16_t*)h, slot_pair, top, (const bf16_t*)gate_up, \
        tile_expert, ff, width, cap, (bf16_t*)mid)
    if (form == EXPERT_GATED_SILU) MOE_UP(1);
    else if (form == EXPERT_GELU) MOE_UP(2);
    else if (form == EXPERT_CAPPED) MOE_UP(3);
    else MOE_UP(4);
#undef MOE_UP
    moe_grouped_kernel<0><<<dim3(max_tiles, (width + GT_FEATURES - 1) / GT_FEATURES), GT_WAVES * WAVE, 0, stream>>>(
        (const bf16_t*)mid, nullptr, top, (const bf16_t*)down, tile_expert, width, ff, cap, (bf16_t*)y);
    moe_combine_kernel<<<n_tokens, combine_threads, 0, stream>>>((const bf16_t*)y, pair_slot, weight, top, width, (const bf16_t*)add0, (const bf16_t*)add1, out);
    PALM_LAUNCHED();
    return 0;
}
