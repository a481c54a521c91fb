// Mixture of experts, gfx950: router, plan of the rows by expert, and the product of sorted rows with their experts'
// weights.  (A decode step of at most 32 rows does not sort: its experts run as batched tah_linear_rows calls, every
// expert that some row chose over all rows.)
//
//  * moe_route_kernel: router logits in float32, their scores, the open groups of experts, the largest ones and their
//    weights; RB rows per workgroup share the router's weights, and a wave takes EB experts at a time so that they share
//    the rows' reads.
//  * moe_plan_kernel: counting sort of the (row, choice) pairs by expert, each expert's rows padded to whole tiles.
//  * moe_tile_kernel: bf16 tiles of 128 places x 256 weight rows on the matrix cores, both operands staged through LDS
//    by asynchronous copies, two stages ahead; gate and up rows of the same columns share a wave, which applies the gate.
//  * moe_plain_kernel: the same product in float32 arithmetic (the float32 form of a model).
#include <hip/hip_runtime.h>

#include "mixer_device.h"

namespace tah {
namespace {

constexpr int kMoeThreads = 256;
constexpr int kMaxExperts = 1024;
constexpr int kMaxTop = 64;
constexpr int kGroupsPerLane = 4;  // groups of experts: at most 256
constexpr int kTile = TAH_MOE_TILE;

// LDS: rows [RB][cols] float32, logits [RB][experts + 1]
template <class X, class E, int RB, int EB, int kThreads>
__global__ __launch_bounds__(kThreads) void moe_route_kernel(const tah_moe_route_args p) {
    HIP_DYNAMIC_SHARED(float, sm)
    const X* const x = static_cast<const X*>(p.x);
    const E* const router = static_cast<const E*>(p.router);
    const E* const gate_w = static_cast<const E*>(p.gate_w);
    const int rows = p.rows, cols = p.cols, experts = p.experts, top = p.top;
    float* const xs = sm;
    float* const z = sm + RB * cols;
    constexpr int kWaves = kThreads / kWave;
    const int tid = threadIdx.x, lane = tid % kWave, wave = tid / kWave, row0 = blockIdx.x * RB;
    const int zs = experts + 1, total = experts + (gate_w ? 1 : 0);
    for (int i = 8 * tid; i < RB * cols; i += 8 * kThreads) {
        const int r = row0 + i / cols;
        float v[8] = {0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f};
        if (r < rows) load8(x + (int64_t)r * cols + i % cols, v);
        store8(xs + i, v);
    }
    __syncthreads();
    for (int e0 = EB * wave; e0 < total; e0 += EB * kWaves) {
        const E* w[EB];
        float s[EB][RB];
#pragma unroll
        for (int x = 0; x < EB; ++x) {
            const int e = e0 + x;
            w[x] = e < experts ? router + (int64_t)e * cols : (e < total ? gate_w : router);  // (past the end: computed, not stored)
#pragma unroll
            for (int r = 0; r < RB; ++r) s[x][r] = 0.f;
        }
        for (int c = 8 * lane; c < cols; c += 8 * kWave) {
            float v[EB][8];
#pragma unroll
            for (int x = 0; x < EB; ++x) load8(w[x] + c, v[x]);
#pragma unroll
            for (int r = 0; r < RB; ++r) {
                float y[8];
                load8(xs + r * cols + c, y);
#pragma unroll
                for (int x = 0; x < EB; ++x)
#pragma unroll
                    for (int i = 0; i < 8; ++i) s[x][r] += v[x][i] * y[i];
            }
        }
#pragma unroll
        for (int x = 0; x < EB; ++x)
#pragma unroll
            for (int r = 0; r < RB; ++r) {
                const float t = wave_sum(s[x][r]);
                if (lane == 0 && e0 + x < total) z[r * zs + e0 + x] = t;
            }
    }
    __syncthreads();
    for (int r = wave; r < RB; r += kWaves) {
        const int row = row0 + r;
        if (row >= rows) break;
        float* const zr = z + r * zs;
        if (gate_w && lane == 0) p.shared_gate[row] = sigmoid_exact(zr[experts]);
        if (p.score == TAH_MOE_SIGMOID) {
            for (int e = lane; e < experts; e += kWave) zr[e] = sigmoid_exact(zr[e]);
            TAH_WAVE_LDS_SYNC();
        }
        if (p.keep < p.groups) {
            // a lane's groups: the sum of their two largest scores; then the best groups one after another, and the others'
            // experts leave the race
            const int size = experts / p.groups;
            float gs[kGroupsPerLane];
#pragma unroll
            for (int u = 0; u < kGroupsPerLane; ++u) {
                const int gr = lane + kWave * u;
                float a = kNegInf, b = kNegInf;
                for (int i = 0; gr < p.groups && i < size; ++i) {
                    const float v = zr[gr * size + i];
                    b = fmaxf(b, fminf(a, v));
                    a = fmaxf(a, v);
                }
                gs[u] = gr < p.groups ? (size > 1 ? a + b : a) : kNegInf;
            }
            uint32_t open = 0;  // bit u: group lane + 64 u is open
            for (int j = 0; j < p.keep; ++j) {
                float bv = kNegInf;
                int bi = 0x7fffffff;
#pragma unroll
                for (int u = 0; u < kGroupsPerLane; ++u)
                    if (!(open >> u & 1) && gs[u] > bv) { bv = gs[u]; bi = lane + kWave * u; }
#pragma unroll
                for (int m = 32; m >= 1; m >>= 1) {
                    const float ov = __shfl_xor(bv, m);
                    const int oi = __shfl_xor(bi, m);
                    if (ov > bv || (ov == bv && oi < bi)) { bv = ov; bi = oi; }
                }
                if (bi % kWave == lane && bi < p.groups) open |= 1u << (bi / kWave);
            }
#pragma unroll
            for (int u = 0; u < kGroupsPerLane; ++u) {
                const int gr = lane + kWave * u;
                for (int i = 0; gr < p.groups && !(open >> u & 1) && i < size; ++i) zr[gr * size + i] = kNegInf;
            }
            TAH_WAVE_LDS_SYNC();
        }
        // the largest scores one after another, the lower index among equals; a chosen one leaves the race
        float mine = kNegInf, first = 0.f;
        int my_index = 0;
        for (int j = 0; j < top; ++j) {
            float bv = kNegInf;
            int bi = 0x7fffffff;
            for (int e = lane; e < experts; e += kWave) {
                const float v = zr[e];
                if (v > bv) { bv = v; bi = e; }
            }
#pragma unroll
            for (int m = 32; m >= 1; m >>= 1) {
                const float ov = __shfl_xor(bv, m);
                const int oi = __shfl_xor(bi, m);
                if (ov > bv || (ov == bv && oi < bi)) { bv = ov; bi = oi; }
            }
            if (bi >= experts) bi = j;  // (only when the logits are not numbers)
            if (j == 0) first = bv;
            if (lane == j) { mine = bv; my_index = bi; }
            if (lane == 0) zr[bi] = kNegInf;
            TAH_WAVE_LDS_SYNC();
        }
        const float w = lane < top ? expf(mine - first) : 0.f;
        const float sum = wave_sum(w);
        if (lane < top) {
            p.index[(int64_t)row * top + lane] = my_index;
            p.weight[(int64_t)row * top + lane] = p.score == TAH_MOE_SIGMOID ? mine : w / sum;
        }
    }
}

constexpr int kPlanThreads = 1024;

__global__ __launch_bounds__(kPlanThreads) void moe_plan_kernel(const int32_t* index, int pairs, int top, int experts, int tiles, int32_t* source,
                                                                int32_t* tile_expert, int32_t* place) {
    __shared__ int32_t count[kMaxExperts], cursor[kMaxExperts], scan[2][kPlanThreads];
    const int tid = threadIdx.x;
    count[tid] = 0;
    __syncthreads();
    for (int i = tid; i < pairs; i += kPlanThreads) atomicAdd(&count[index[i]], 1);
    __syncthreads();
    const int n = count[tid], mine = (n + kTile - 1) / kTile;
    int from = 0;
    scan[0][tid] = mine;
    __syncthreads();
    for (int d = 1; d < kPlanThreads; d <<= 1) {
        scan[from ^ 1][tid] = scan[from][tid] + (tid >= d ? scan[from][tid - d] : 0);
        from ^= 1;
        __syncthreads();
    }
    const int t0 = scan[from][tid] - mine, used = scan[from][kPlanThreads - 1];
    cursor[tid] = t0 * kTile;
    for (int t = 0; t < mine; ++t) tile_expert[t0 + t] = tid;
    for (int i = n; i < mine * kTile; ++i) source[t0 * kTile + i] = -1;
    for (int t = used + tid; t < tiles; t += kPlanThreads) tile_expert[t] = -1;
    if (tid == 0) tile_expert[tiles] = used;
    __syncthreads();
    for (int i = tid; i < pairs; i += kPlanThreads) {
        const int at = atomicAdd(&cursor[index[i]], 1);
        source[at] = i / top;
        place[i] = at;
    }
}

struct MoeGemm {
    const void* x;
    const void* w;
    const int32_t *source, *tile_expert;
    void* out;
    int64_t x_rs, out_rs;
    int32_t n, k, tiles, col_tiles, act;
    float c0, c1;
};

// Which tile of places and which tile of columns a workgroup takes.  Workgroups go to the XCDs round robin; an XCD gets a
// run of consecutive place tiles with all their columns, so that an expert's weights and a place's row are read into
// one L2 only.  False: nothing to do.
__device__ __forceinline__ bool moe_tile_of(const MoeGemm& p, int item, int& tile, int& col_tile) {
    const int used = const_i32(p.tile_expert, p.tiles), per = (used + 7) / 8;
    const int xcd = item % 8, i = item / 8;
    tile = xcd * per + i / p.col_tiles;
    col_tile = i % p.col_tiles;
    return i / p.col_tiles < per && tile < used;
}

// ---- bf16 tiles ------------------------------------------------------------------------------------------------
constexpr int kStageK = 64;     // a whole 128-byte line of every row per stage
constexpr int kStages = 3;
constexpr int kTileW = 256;     // weight rows of a tile
constexpr int kTileWaves = 8;
constexpr int kTileWalkers = 256;  // workgroups: one per compute unit
constexpr int kStageBytes = (kTile + kTileW) * kStageK * 2;

// A workgroup walks tiles blockIdx.x, blockIdx.x + gridDim.x, ... (gridDim.x % 8 == 0: all of one XCD) as one run of stages:
// the first stages of the next tile are on their way while the last ones of this tile are multiplied and its result is
// written.  Eight waves, 2 x 4: wave (wm, wn) computes places 64 wm ... + 63 against weight rows 64 wn ... + 63 of the tile.
template <bool GATE>
__global__ __launch_bounds__(kTileWaves * kWave) void moe_tile_kernel(const MoeGemm p) {
    HIP_DYNAMIC_SHARED(unsigned char, lds)
    const int lane = threadIdx.x % kWave, wave = __builtin_amdgcn_readfirstlane(threadIdx.x / kWave), wm = wave / 4, wn = wave % 4;
    const __bf16* const x = static_cast<const __bf16*>(p.x);
    constexpr int kCols = GATE ? kTileW / 2 : kTileW;  // output columns of a tile
    int tile, col_tile;
    if (!moe_tile_of(p, blockIdx.x, tile, col_tile)) return;  // (an XCD's tiles come without gaps: nothing here, nothing further on)
    int item = blockIdx.x, next = blockIdx.x;  // the tile being multiplied, and the one the copies are at
    __bf16* const out = static_cast<__bf16*>(p.out);
    // This lane's part of the copies: of every eight rows a wave copies, row lane / 8, sixteen bytes at logical chunk
    // (lane % 8) ^ swizzle(row) -- the chunks of a row lie permuted in LDS so that the operand reads do not collide.
    constexpr int kA = kTile / 8 / kTileWaves, kB = kTileW / 8 / kTileWaves;  // copies per wave and stage: 2 and 4
    const __bf16 *ga[kA], *gb[kB];
    const int chunk = (lane % 8) ^ ((lane / 16) & 7);  // ((row >> 1) & 7 with row = 8 i + lane / 8: i's part is even)
    auto point_at = [&](int tl, int ct) __attribute__((always_inline)) {
        const __bf16* const w = static_cast<const __bf16*>(p.w) + (int64_t)const_i32(p.tile_expert, tl) * (GATE ? 2 : 1) * p.n * p.k;
        const int c0 = ct * kCols;
#pragma unroll
        for (int i = 0; i < kA; ++i) {
            const int r = 8 * (kA * wave + i) + lane / 8;
            int src = GATE ? p.source[tl * kTile + r] : tl * kTile + r;
            src = src < 0 ? 0 : src;  // a padding place computes row 0 again; nobody reads it
            ga[i] = x + (int64_t)src * p.x_rs;
        }
#pragma unroll
        for (int i = 0; i < kB; ++i) {
            const int r = 8 * (kB * wave + i) + lane / 8;
            int wr;
            if constexpr (GATE) {  // rows of the tile: 32 gate, 32 up of the first 32 columns, then of the next
                int c = c0 + 32 * (r / 64) + r % 32;
                c = c < p.n ? c : p.n - 1;
                wr = (r / 32) % 2 ? p.n + c : c;
            } else {
                wr = c0 + r < p.n ? c0 + r : p.n - 1;
            }
            gb[i] = w + (int64_t)wr * p.k;
        }
    };
    point_at(tile, col_tile);
    const int stages = (p.k + kStageK - 1) / kStageK;
    int ahead = 0, slot = 0;  // the stage of that tile the next copies are for, and their place in LDS
    bool open = true;         // there is one
    int pending = 0;          // stages whose copies are under way or in, not yet multiplied
    auto stage = [&]() __attribute__((always_inline)) {
        if (!open) return;
        if (ahead == stages) {
            int tl, ct;
            next += gridDim.x;
            open = moe_tile_of(p, next, tl, ct);
            if (!open) return;
            point_at(tl, ct);
            ahead = 0;
        }
        ++pending;
        const int s = ahead++;
        unsigned char* const base = lds + slot * kStageBytes;
        slot = slot + 1 < kStages ? slot + 1 : 0;
        const int k0 = s * kStageK, valid = (p.k - k0) / 8;  // chunks of this stage inside the rows
#pragma unroll
        for (int i = 0; i < kA; ++i) {
            const int c = chunk ^ ((4 * (kA * wave + i)) & 7);
            async_copy_16B(ga[i] + k0 + 8 * (c < valid ? c : 0), base + (kA * wave + i) * 1024);
        }
#pragma unroll
        for (int i = 0; i < kB; ++i) {
            const int c = chunk ^ ((4 * (kB * wave + i)) & 7);
            async_copy_16B(gb[i] + k0 + 8 * (c < valid ? c : 0), base + kTile * kStageK * 2 + (kB * wave + i) * 1024);
        }
    };
    f32x4 acc[4][4];  // [weight tile][place tile]
#pragma unroll
    for (int i = 0; i < 4; ++i)
#pragma unroll
        for (int j = 0; j < 4; ++j) acc[i][j] = f32x4{0.f, 0.f, 0.f, 0.f};
    for (int s = 0; s < kStages - 1; ++s) stage();
    int done = 0, at = 0;  // stages of `tile` that are multiplied; where the next one lies in LDS
    while (pending > 0) {
        // all but the copies of the one stage behind this one have landed (and the stores of a finished tile)
        if (pending >= 2) TAH_WAIT_VMEM_N(kA + kB);
        else TAH_WAIT_VMEM();
        __syncthreads();  // every wave's copies of this stage are in, and nobody reads the one before any more
        --pending;
        stage();
        const int s = done++;
        const unsigned char* const a = lds + at * kStageBytes;
        at = at + 1 < kStages ? at + 1 : 0;
        const unsigned char* const b = a + kTile * kStageK * 2;
        auto multiply = [&](int h) __attribute__((always_inline)) {
            bf16x8 fx[4], fw[4];
#pragma unroll
            for (int j = 0; j < 4; ++j) fx[j] = *reinterpret_cast<const bf16x8*>(a + rowmajor64_off(64 * wm + 16 * j + lane % 16, 4 * h + lane / 16));
#pragma unroll
            for (int i = 0; i < 4; ++i) fw[i] = *reinterpret_cast<const bf16x8*>(b + rowmajor64_off(64 * wn + 16 * i + lane % 16, 4 * h + lane / 16));
#pragma unroll
            for (int i = 0; i < 4; ++i)
#pragma unroll
                for (int j = 0; j < 4; ++j) acc[i][j] = mfma16(fw[i], fx[j], acc[i][j]);
        };
        multiply(0);
        if (s * kStageK + 32 < p.k) multiply(1);  // (uniform)
        if (done < stages) continue;
        // accumulator (i, j) register r of lane l: weight row 16 i + 4 (l / 16) + r, place 16 j + l % 16
        const int n0 = col_tile * kCols;
#pragma unroll
        for (int j = 0; j < 4; ++j) {
            __bf16* const row = out + ((int64_t)tile * kTile + 64 * wm + 16 * j + lane % 16) * p.out_rs;
            if constexpr (GATE) {
#pragma unroll
                for (int i = 0; i < 2; ++i) {
                    const int c = n0 + 32 * wn + 16 * i + 4 * (lane / 16);
                    bf16x4 y;
#pragma unroll
                    for (int r = 0; r < 4; ++r)
                        y[r] = (__bf16)(p.act == TAH_ACT_CLAMPED_GATE ? clamped_gate(acc[i][j][r], acc[2 + i][j][r], p.c0, p.c1)
                                                                      : (acc[i][j][r] / (1.0f + fast_exp2(-acc[i][j][r] * kLog2e))) * acc[2 + i][j][r]);
                    if (c < p.n) *reinterpret_cast<bf16x4*>(row + c) = y;
                }
            } else {
#pragma unroll
                for (int i = 0; i < 4; ++i) {
                    const int c = n0 + 64 * wn + 16 * i + 4 * (lane / 16);
                    bf16x4 y;
#pragma unroll
                    for (int r = 0; r < 4; ++r) y[r] = (__bf16)acc[i][j][r];
                    if (c < p.n) *reinterpret_cast<bf16x4*>(row + c) = y;
                }
            }
        }
#pragma unroll
        for (int i = 0; i < 4; ++i)
#pragma unroll
            for (int j = 0; j < 4; ++j) acc[i][j] = f32x4{0.f, 0.f, 0.f, 0.f};
        done = 0;
        item += gridDim.x;
        if (!moe_tile_of(p, item, tile, col_tile)) return;
    }
}

// ---- float32 ---------------------------------------------------------------------------------------------------
constexpr int kPlainK = 16, kPlainCols = 32;

// 128 places x 32 columns per workgroup; thread (column tid % 32, places tid / 32 + 8 i)
template <bool GATE>
__global__ __launch_bounds__(kMoeThreads) void moe_plain_kernel(const MoeGemm p) {
    __shared__ float a[kPlainK][kTile + 1], g[kPlainK][kPlainCols + 1], u[GATE ? kPlainK : 1][kPlainCols + 1];
    int tile, col_tile;
    if (!moe_tile_of(p, blockIdx.x, tile, col_tile)) return;
    const int expert = p.tile_expert[tile];
    const int tid = threadIdx.x, tc = tid % kPlainCols, tr = tid / kPlainCols, n0 = col_tile * kPlainCols;
    const float* const x = static_cast<const float*>(p.x);
    const float* const w = static_cast<const float*>(p.w) + (int64_t)expert * (GATE ? 2 : 1) * p.n * p.k;
    float sg[16], su[16];
#pragma unroll
    for (int i = 0; i < 16; ++i) sg[i] = su[i] = 0.f;
    for (int k0 = 0; k0 < p.k; k0 += kPlainK) {
        for (int i = tid; i < kTile * kPlainK; i += kMoeThreads) {
            const int r = i / kPlainK, c = i % kPlainK;
            const int src = GATE ? p.source[tile * kTile + r] : tile * kTile + r;
            a[c][r] = src >= 0 ? x[(int64_t)src * p.x_rs + k0 + c] : 0.f;
        }
        for (int i = tid; i < kPlainCols * kPlainK; i += kMoeThreads) {
            const int r = i / kPlainK, c = i % kPlainK, wr = n0 + r < p.n ? n0 + r : p.n - 1;
            g[c][r] = w[(int64_t)wr * p.k + k0 + c];
            if constexpr (GATE) u[c][r] = w[((int64_t)p.n + wr) * p.k + k0 + c];
        }
        __syncthreads();
#pragma unroll
        for (int c = 0; c < kPlainK; ++c) {
            const float wg = g[c][tc], wu = GATE ? u[GATE ? c : 0][tc] : 0.f;
#pragma unroll
            for (int i = 0; i < 16; ++i) {
                const float v = a[c][tr + 8 * i];
                sg[i] += v * wg;
                if constexpr (GATE) su[i] += v * wu;
            }
        }
        __syncthreads();
    }
    if (n0 + tc >= p.n) return;
#pragma unroll
    for (int i = 0; i < 16; ++i)
        static_cast<float*>(p.out)[((int64_t)tile * kTile + tr + 8 * i) * p.out_rs + n0 + tc] =
            !GATE ? sg[i] : (p.act == TAH_ACT_CLAMPED_GATE ? clamped_gate_exact(sg[i], su[i], p.c0, p.c1) : silu_exact(sg[i]) * su[i]);
}

template <class X, class E>
void launch_route(const tah_moe_route_args& a, hipStream_t st) {
    const auto lds = [&](int rb) { return (size_t)rb * (a.cols + a.experts + 1) * sizeof(float); };
    if (a.rows > 256 && lds(4) <= 65536)  // many rows: four share a pass over the router's weights
        hipLaunchKernelGGL((moe_route_kernel<X, E, 4, 4, 256>), dim3((a.rows + 3) / 4), dim3(256), lds(4), st, a);
    else  // few rows: what counts is how much of the router's weights one row has in flight
        hipLaunchKernelGGL((moe_route_kernel<X, E, 1, 2, 1024>), dim3(a.rows), dim3(1024), lds(1), st, a);
}

int tile_capacity(int64_t pairs, int experts) { return (int)(pairs / kTile + (experts < pairs ? experts : pairs)); }

}  // namespace
}  // namespace tah

extern "C" int tah_moe_route(const tah_moe_route_args* a, tah_stream_t stream) {
    using namespace tah;
    if (!a) return TAH_E_NULL;
    if (a->rows < 0 || a->cols <= 0 || a->cols % 8 != 0 || a->experts <= 0 || a->experts > kMaxExperts || a->top <= 0 || a->top > kMaxTop ||
        a->top > a->experts || (a->dtype != TAH_DT_BF16 && a->dtype != TAH_DT_F32) || (a->score != TAH_MOE_SOFTMAX && a->score != TAH_MOE_SIGMOID))
        return TAH_E_SHAPE;
    if (a->groups <= 0 || a->groups > kWave * kGroupsPerLane || a->experts % a->groups != 0 || a->keep <= 0 || a->keep > a->groups ||
        a->top > a->experts / a->groups * a->keep)
        return TAH_E_SHAPE;
    if ((size_t)(a->cols + a->experts + 1) * sizeof(float) > 65536) return TAH_E_SHAPE;
    if (a->rows == 0) return TAH_OK;
    if (!a->x || !a->router || !a->index || !a->weight || (a->gate_w && !a->shared_gate)) return TAH_E_NULL;
    if (!aligned_16(a->x) || !aligned_16(a->router) || !aligned_16(a->gate_w)) return TAH_E_ALIGN;
    hipStream_t st = static_cast<hipStream_t>(stream);
    if (a->dtype == TAH_DT_F32) launch_route<float, float>(*a, st);
    else if (a->x_elem) launch_route<__bf16, __bf16>(*a, st);
    else launch_route<float, __bf16>(*a, st);
    return launch_status();
}

extern "C" int32_t tah_moe_places(int32_t rows, int32_t top, int32_t experts) {
    return rows <= 0 || top <= 0 || experts <= 0 ? 0 : tah::tile_capacity((int64_t)rows * top, experts) * TAH_MOE_TILE;
}

extern "C" int tah_moe_plan(const int32_t* index, int32_t rows, int32_t top, int32_t experts, int32_t* source, int32_t* tile_expert, int32_t* place,
                            tah_stream_t stream) {
    using namespace tah;
    if (rows < 0 || top <= 0 || top > kMaxTop || experts <= 0 || experts > kMaxExperts || (int64_t)rows * top > (1 << 30)) return TAH_E_SHAPE;
    if (rows == 0) return TAH_OK;
    if (!index || !source || !tile_expert || !place) return TAH_E_NULL;
    hipLaunchKernelGGL(moe_plan_kernel, dim3(1), dim3(kPlanThreads), 0, static_cast<hipStream_t>(stream), index, (int)(rows * top), (int)top,
                       (int)experts, tile_capacity((int64_t)rows * top, experts), source, tile_expert, place);
    return launch_status();
}

extern "C" int tah_moe_linear(const void* x, int64_t x_rs, const void* w, const int32_t* source, const int32_t* tile_expert, int32_t tiles, int32_t n,
                              int32_t k, int32_t kind, int32_t activation, float c0, float c1, void* out, int64_t out_rs, int32_t dtype,
                              tah_stream_t stream) {
    using namespace tah;
    if (tiles < 0 || tiles > 65535 || n <= 0 || k <= 0 || n % 4 != 0 || k % 32 != 0 || x_rs < k || out_rs < n || x_rs % 8 != 0 || out_rs % 4 != 0 ||
        (kind != TAH_LINEAR_PLAIN && kind != TAH_LINEAR_GATE_UP) || (activation != TAH_ACT_NONE && activation != TAH_ACT_CLAMPED_GATE) ||
        (dtype != TAH_DT_BF16 && dtype != TAH_DT_F32))
        return TAH_E_SHAPE;
    if (tiles == 0) return TAH_OK;
    if (!x || !w || !tile_expert || !out || (kind == TAH_LINEAR_GATE_UP && !source)) return TAH_E_NULL;
    if (!aligned_16(x) || !aligned_16(w) || !aligned_16(out)) return TAH_E_ALIGN;
    const bool gate = kind == TAH_LINEAR_GATE_UP;
    const int cols = dtype == TAH_DT_F32 ? kPlainCols : (gate ? kTileW / 2 : kTileW);
    const MoeGemm p{x, w, source, tile_expert, out, x_rs, out_rs, n, k, tiles, (n + cols - 1) / cols, activation, c0, c1};
    const int64_t groups = (int64_t)((tiles + 7) / 8) * 8 * p.col_tiles;  // whole rounds over the XCDs
    if (groups > 0x7fffffff) return TAH_E_SHAPE;
    const dim3 grid((unsigned)groups);
    hipStream_t st = static_cast<hipStream_t>(stream);
    if (dtype == TAH_DT_BF16) {
        const void* f = gate ? reinterpret_cast<const void*>(&moe_tile_kernel<true>) : reinterpret_cast<const void*>(&moe_tile_kernel<false>);
        if (hipFuncSetAttribute(f, hipFuncAttributeMaxDynamicSharedMemorySize, kStages * kStageBytes) != hipSuccess) return TAH_E_LAUNCH;
        // (walking pays where a tile is few stages, behind an expert's hidden size; the long tiles of gate|up lose a little by it)
        const dim3 walk((unsigned)(gate || groups < kTileWalkers ? groups : kTileWalkers));
        if (gate) hipLaunchKernelGGL((moe_tile_kernel<true>), walk, dim3(kTileWaves * kWave), kStages * kStageBytes, st, p);
        else hipLaunchKernelGGL((moe_tile_kernel<false>), walk, dim3(kTileWaves * kWave), kStages * kStageBytes, st, p);
    } else {
        if (gate) hipLaunchKernelGGL((moe_plain_kernel<true>), grid, dim3(kMoeThreads), 0, st, p);
        else hipLaunchKernelGGL((moe_plain_kernel<false>), grid, dim3(kMoeThreads), 0, st, p);
    }
    return launch_status();
}
