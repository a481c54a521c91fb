// Attention in a sliding window with kept first tokens, grouped query heads, rotary positions on part of a head, and one
// gate per head, gfx950.  A token's keys and values of one key/value head are one cached row, the values its first columns
// and the keys its last ones; where the keys (before rotation) are the values, the two overlap and the row is hardly longer
// than either.  A slot keeps its first tokens and a ring as long as the window.
//
//  * window_prep_kernel: rotates queries and keys of a step's rows in place (and enters single tokens into the cache).
//  * window_tile_kernel (bf16): portions.  Four waves, 16 queries x 2 each, of all query heads of one key/value head, so that
//    one pass over its keys (64 rows at a time, in LDS once for keys and values) serves them all; S^T = K Q^T and O^T =
//    V^T P^T, V^T read from the row-major tile by transpose reads.  Keys before the portion come from the cache, its own
//    from the projections; tiles outside the window and behind the kept tokens are not visited.
//  * window_append_kernel: a portion's rows into the cache.
//  * window_decode_kernel (bf16): single tokens.  Rotation, cache entry and attention in one launch: every wave takes 32 keys
//    at a time with a softmax state of its own (no barrier until the end), all query heads of one key/value head share
//    the pass.  A call with few rows splits the keys over workgroups; window_merge_kernel adds the parts.
//  * window_rows_kernel: one workgroup per (query, head), any sizes, either element type (the float32 form).
//
// Scores, weights and sums are float32.  Where a weight enters a bf16 matrix product it goes in as two bf16 terms
// (its rounding and what the rounding left), so that it keeps sixteen bits.
#include <hip/hip_runtime.h>

#include "mixer_device.h"

namespace tah {
namespace {

constexpr int kWinThreads = 256;
constexpr int kWinWaves = kWinThreads / kWave;

// Rows of one slot's and head's cache, addressed by position.  Positions asked for together lie in [lo, lo + ring), where lo is
// what the view was made for, or below keep: so at most one wrap, and one division when the view is made.
struct RingView {
    int keep, ring, shift;
    __device__ __forceinline__ RingView(int keep_, int ring_, int lo) : keep(keep_), ring(ring_) {
        shift = keep + (lo > keep ? (lo - keep) / ring * ring : 0);
    }
    __device__ __forceinline__ int row(int pos) const {
        int r = pos - shift;
        r = r >= ring ? r - ring : r;
        return pos < keep ? pos : keep + r;
    }
};

// ---- rotation ----------------------------------------------------------------------------------------------------
// grid (rows); pairs of all heads, then (with a slot) the rows into the cache
template <class E>
__global__ __launch_bounds__(kWinThreads) void window_prep_kernel(const tah_window_layer L, const tah_window_rows R) {
    const int row = blockIdx.x, tid = threadIdx.x;
    E* const pr = static_cast<E*>(R.proj) + (int64_t)row * R.proj_row_stride;
    const int p0 = R.pos[row], pos = p0 < 0 ? 0 : (p0 >= R.table_rows ? R.table_rows - 1 : p0);
    const int half = L.rot_dim / 2;
    const float* const co = R.cos + (int64_t)pos * half;
    const float* const si = R.sin + (int64_t)pos * half;
    for (int i = tid; i < (L.heads + L.kv_heads) * half; i += kWinThreads) {
        const int h = i / half, m = i % half;
        const E* src;
        E* dst;
        if (h < L.heads) {
            dst = pr + R.q_col + h * L.key_dim + L.key_dim - L.rot_pad + 2 * m;
            src = dst;
        } else {
            E* const r = pr + R.k_col + (h - L.heads) * L.row;
            dst = r + L.row - L.rot_pad + 2 * m;
            src = r + L.rot_source + 2 * m;
        }
        const float u = (float)src[0], v = (float)src[1];
        dst[0] = (E)(u * co[m] - v * si[m]);
        dst[1] = (E)(v * co[m] + u * si[m]);
    }
    const int slot = R.slot ? R.slot[row] : -1;
    if (slot < 0 || slot >= L.nslots || p0 < 0) return;
    __syncthreads();
    const int at = p0 < L.keep_first ? p0 : L.keep_first + (p0 - L.keep_first) % L.ring, span = L.keep_first + L.ring;
    for (int i = 8 * tid; i < L.kv_heads * L.row; i += 8 * kWinThreads) {
        const int g = i / L.row, c = i % L.row;
        float v[8];
        load8(pr + R.k_col + i, v);
        store8(static_cast<E*>(L.cache) + (((int64_t)slot * L.kv_heads + g) * span + at) * L.row + c, v);
    }
}

// one wave per row of the portions
template <class E>
__global__ __launch_bounds__(kWinThreads) void window_append_kernel(const tah_window_layer L, const tah_portions P, const tah_window_rows R) {
    const int lane = threadIdx.x % kWave, row = blockIdx.x * kWinWaves + threadIdx.x / kWave;
    if (row >= P.rows) return;
    const int b = P.row_seq[row], slot = P.slot[b];
    if (slot < 0 || slot >= L.nslots) return;
    const int pos = P.pos0[b] + row - P.cu[b];
    if (pos >= L.keep_first && P.cu[b + 1] - row > L.ring) return;  // (overwritten by a later row of the portion)
    const int at = pos < L.keep_first ? pos : L.keep_first + (pos - L.keep_first) % L.ring, span = L.keep_first + L.ring;
    const E* const src = static_cast<const E*>(R.proj) + (int64_t)row * R.proj_row_stride + R.k_col;
    for (int i = 8 * lane; i < L.kv_heads * L.row; i += 8 * kWave) {
        const int g = i / L.row, c = i % L.row;
        float v[8];
        load8(src + i, v);
        store8(static_cast<E*>(L.cache) + (((int64_t)slot * L.kv_heads + g) * span + at) * L.row + c, v);
    }
}

// ---- any sizes, either element type: one workgroup per (query row, head) ----------------------------------------
struct WindowCall {
    tah_window_layer L;
    tah_window_rows R;
    tah_portions P;       // nseq 0: single tokens, every key in the cache
    void* out;
    void* out_packed;
    int64_t out_rs;
};

constexpr int kRowKeys = 64;    // keys per pass
constexpr int kRowValues = 4;   // value elements per thread: value_dim <= 1024

template <class E>
__global__ __launch_bounds__(kWinThreads) void window_rows_kernel(const WindowCall p) {
    HIP_DYNAMIC_SHARED(float, qs)   // [key_dim]
    __shared__ float sc[kRowKeys];
    const tah_window_layer& L = p.L;
    const tah_window_rows& R = p.R;
    const int row = blockIdx.x, h = blockIdx.y, tid = threadIdx.x, lane = tid % kWave, wave = tid / kWave;
    const int g = h / (L.heads / L.kv_heads), span = L.keep_first + L.ring;
    int pos, slot, pos0;  // pos0: keys from here on are projections' rows
    int64_t own = 0;      // row of the projections that is position 0's
    if (p.P.nseq == 0) {
        pos = R.pos[row];
        slot = R.slot[row];
        pos0 = 0x7fffffff;
    } else {
        const int b = p.P.row_seq[row];
        pos0 = p.P.pos0[b];
        pos = pos0 + row - p.P.cu[b];
        slot = p.P.slot[b];
        own = (int64_t)p.P.cu[b] - pos0;
    }
    if (slot >= L.nslots) slot = -1;
    const bool live = pos >= 0 && (slot >= 0 || p.P.nseq != 0);
    const E* const proj = static_cast<const E*>(R.proj);
    const E* const q = proj + (int64_t)row * R.proj_row_stride + R.q_col + h * L.key_dim;
    const E* const cache = static_cast<const E*>(L.cache) + ((int64_t)(slot < 0 ? 0 : slot) * L.kv_heads + g) * span * L.row;
    int lo = pos - L.window + 1;
    lo = lo < 0 ? 0 : lo;
    const RingView view(L.keep_first, L.ring, lo);
    const int kept = L.keep_first < lo ? L.keep_first : lo, nk = live ? kept + pos - lo + 1 : 0;  // kept first tokens, then the window
    auto key = [&](int x) __attribute__((always_inline)) {
        const int j = x < kept ? x : lo + x - kept;
        return j >= pos0 ? proj + (own + j) * R.proj_row_stride + R.k_col + g * L.row : cache + (int64_t)view.row(j) * L.row;
    };
    for (int i = tid; i < L.key_dim; i += kWinThreads) qs[i] = (float)q[i];
    __syncthreads();
    float acc[kRowValues], m = kNoScore, l = 0.f;
#pragma unroll
    for (int e = 0; e < kRowValues; ++e) acc[e] = 0.f;
    for (int x0 = 0; x0 < nk; x0 += kRowKeys) {
        for (int x = wave; x < kRowKeys; x += kWinWaves) {
            float s = 0.f;
            if (x0 + x < nk) {
                const E* const k = key(x0 + x) + L.row - L.key_dim;
                for (int i = lane; i < L.key_dim; i += kWave) s += qs[i] * (float)k[i];
            }
            s = wave_sum(s);
            if (lane == 0) sc[x] = x0 + x < nk ? s * L.scale : kNegInf;
        }
        __syncthreads();
        const float mn = fmaxf(m, wave_max(sc[lane]));
        const float a = expf(m - mn);
        m = mn;
        l = l * a + wave_sum(expf(sc[lane] - m));
#pragma unroll
        for (int e = 0; e < kRowValues; ++e) acc[e] *= a;
        const int n = nk - x0 < kRowKeys ? nk - x0 : kRowKeys;
        for (int x = 0; x < n; ++x) {
            const float w = expf(sc[x] - m);
            const E* const v = key(x0 + x);
#pragma unroll
            for (int e = 0; e < kRowValues; ++e) {
                const int i = tid + e * kWinThreads;
                if (i < L.value_dim) acc[e] += w * (float)v[i];
            }
        }
        __syncthreads();
    }
    const float gate = R.g_col >= 0 ? sigmoid_exact((float)proj[(int64_t)row * R.proj_row_stride + R.g_col + h]) : 1.0f;
#pragma unroll
    for (int e = 0; e < kRowValues; ++e) {
        const int i = tid + e * kWinThreads;
        if (i >= L.value_dim) continue;
        const float y = live ? acc[e] / l * gate : 0.f;
        if (p.out) static_cast<E*>(p.out)[row * p.out_rs + h * L.value_dim + i] = (E)y;
        if (p.out_packed) static_cast<__bf16*>(p.out_packed)[rows_form_elem(row, h * L.value_dim + i)] = (__bf16)y;
    }
}

// ---- portions on the matrix cores --------------------------------------------------------------------------------
constexpr int kTileKeys = 64;
constexpr int kTileWaves = 4;  // (two workgroups of four run better side by side than one of eight: their barriers differ)
constexpr int kTileThreads = kTileWaves * kWave;
constexpr int kTileQueries = 2 * kTileWaves;  // tiles of 16 queries of one head
constexpr int kTileRows = 8 * kTileKeys / kTileThreads;  // rows of a key tile per thread, eight threads to a row

// Row stride of a tile in LDS: an odd multiple of 16 elements, so that eight rows' same sixteen elements lie in different
// banks; the sixteen-byte units of a pair change places in every other eight rows, so that one unit of sixteen rows does too.
__device__ __host__ __forceinline__ int tile_stride(int row) { return (row + 15) / 32 * 32 + 16; }
__device__ __forceinline__ int tile_unit(int row, int stride, int unit) { return row * stride + 8 * (unit ^ ((row >> 3) & 1)); }

constexpr float kSlack = 8.0f;  // in powers of two

struct WindowTile {
    WindowCall c;
    int32_t slots, per_xcd, chunks, heads_per_tile;  // a key/value head's query heads in chunks of so many
    float scale_log2;
};

// NQ: 32-wide steps of a key (at most), NV: 16-wide tiles of a value row (at most; kExact: just so many), NU: 16-byte units of
// a key tile per thread (at most; eight threads to a row).
template <int NQ, int NV, int NU, bool kExact>
__global__ __launch_bounds__(kTileThreads) TAH_WAVES_PER_EU(NQ <= 4 ? 2 : 1, 8) void window_tile_kernel(const WindowTile p) {
    HIP_DYNAMIC_SHARED(unsigned char, tile_lds)
    const tah_window_layer& L = p.c.L;
    const tah_window_rows& R = p.c.R;
    // (workgroups go to the XCDs round robin: an XCD gets a run of tiles, head by head, whose keys then share its L2)
    const int item = blockIdx.x % 8 * p.per_xcd + blockIdx.x / 8;
    int tile = item % p.slots, b = 0, row0 = 0, row_end = 0;
    const int gc = item / p.slots, g = gc / p.chunks, per = L.heads / L.kv_heads;
    if (g >= L.kv_heads) return;
    const int hpt = p.heads_per_tile, h0 = g * per + (gc % p.chunks) * hpt, h_end = (g + 1) * per;
    const int ptiles = kTileQueries / hpt;  // tiles of 16 positions
    if (!find_tile(p.c.P.cu, p.c.P.nseq, 16 * ptiles, tile, b, row0, row_end)) return;
    const int tid = threadIdx.x, lane = tid % kWave, wave = tid / kWave, c = lane % 16, gq = lane / 16;
    const int nq = kExact ? NQ : L.key_dim / 32, nv = kExact ? NV : L.value_dim / 16;
    const int ks = tile_stride(L.row), koff = L.row - L.key_dim;
    __bf16* const kt = reinterpret_cast<__bf16*>(tile_lds);
    const int buffer = kTileKeys * ks;  // two of them: the next tile is written while this one is read
    const int first = p.c.P.cu[b], pos0 = p.c.P.pos0[b], shift = pos0 - first;  // position of a row: row + shift
    const int slot = p.c.P.slot[b];
    const __bf16* const proj = static_cast<const __bf16*>(R.proj);
    bf16x8 q[2][NQ];
    int own[2], head[2], qrow[2];
    bool on[2];
#pragma unroll
    for (int t = 0; t < 2; ++t) {
        const int u = 2 * wave + t, pt = u / hpt;
        head[t] = h0 + u % hpt;
        on[t] = pt < ptiles && head[t] < h_end;
        if (!on[t]) head[t] = h0;
        int r = row0 + 16 * (pt < ptiles ? pt : 0) + c;
        qrow[t] = r;
        on[t] = on[t] && r < row_end;
        r = r < row_end ? r : row_end - 1;  // rows past the end repeat the last one and are not stored
        own[t] = r + shift;
#pragma unroll
        for (int s = 0; s < NQ; ++s)
            if (kExact || s < nq)
                q[t][s] = *reinterpret_cast<const bf16x8*>(proj + (int64_t)r * R.proj_row_stride + R.q_col + head[t] * L.key_dim + 32 * s + 8 * gq);
    }
    // positions of this wave's queries, and of the workgroup's
    int own_lo = own[0] < own[1] ? own[0] : own[1], own_hi = own[0] < own[1] ? own[1] : own[0];
    own_lo = __builtin_amdgcn_readfirstlane(wave_reduce_min(own_lo));
    own_hi = __builtin_amdgcn_readfirstlane(wave_reduce_max(own_hi));
    const bool busy = __ballot(on[0] || on[1]) != 0;
    int j_lo = row0 + shift - L.window + 1;
    j_lo = j_lo < 0 ? 0 : j_lo;
    const int j_hi = row_end - 1 + shift;
    const int keep = L.keep_first, kept = keep < j_lo ? keep : j_lo;  // kept tokens in front of the window's keys
    const RingView view(keep, L.ring, j_lo);
    f32x4 acc[NV][2];
    f32x4 l[2] = {f32x4{0.f, 0.f, 0.f, 0.f}, f32x4{0.f, 0.f, 0.f, 0.f}};
    float m[2] = {kNoScore, kNoScore};
    bf16x8 ones;
#pragma unroll
    for (int i = 0; i < 8; ++i) ones[i] = (__bf16)1.0f;
#pragma unroll
    for (int i = 0; i < NV; ++i)
#pragma unroll
        for (int t = 0; t < 2; ++t) acc[i][t] = f32x4{0.f, 0.f, 0.f, 0.f};
    const int units = L.row / 8;
    const __bf16* const mine = proj + R.k_col + g * L.row;
    const __bf16* const cache = static_cast<const __bf16*>(L.cache) +
                                ((int64_t)(slot < 0 || slot >= L.nslots ? 0 : slot) * L.kv_heads + g) * (keep + L.ring) * L.row;
    // operand addresses: of K, row 16 x + c, unit koff / 8 + 4 s + gq; of V^T, rows 16 x + 4 gq + c / 4, elements 16 i + 4 (c % 4)
    // (koff % 16 == 0: a unit's partner is not in another pair)
    const int k_at = c * ks + koff + 8 * (gq ^ (c >> 3)), v_at = (4 * gq + c / 4) * ks + 8 * ((c % 4 / 2) ^ (gq >> 1)) + 4 * (c % 2);
    const int fkey = tid / 8, fu = tid % 8;  // this thread's rows fkey + kTileKeys / kTileRows * r, and units fu, fu + 8, ... of them
    constexpr int kRowStep = kTileKeys / kTileRows;
    bf16x8 f[kTileRows][NU];
    // Tiles of keys: those of the kept tokens, [0, kept), then the window's, [j_lo, j_hi], at multiples of 64 positions.  A
    // place outside these repeats the nearest key inside (its score is masked).
    const int kept_tiles = (kept + kTileKeys - 1) / kTileKeys, t_lo = j_lo / kTileKeys, t_hi = j_hi / kTileKeys;
    const int tiles = kept_tiles + t_hi - t_lo + 1;
    auto first_key = [&](int it) __attribute__((always_inline)) { return (it < kept_tiles ? it : it - kept_tiles + t_lo) * kTileKeys; };
    auto fetch = [&](int it) __attribute__((always_inline)) {
        const int j0 = first_key(it), lo = it < kept_tiles ? 0 : j_lo, hi = it < kept_tiles ? kept - 1 : j_hi;
#pragma unroll
        for (int r = 0; r < kTileRows; ++r) {
            int j = j0 + fkey + kRowStep * r;
            j = j < lo ? lo : (j > hi ? hi : j);
            const __bf16* const src = (j >= pos0 ? mine + (int64_t)(j - shift) * R.proj_row_stride : cache + (int64_t)view.row(j) * L.row) + 8 * fu;
#pragma unroll
            for (int i = 0; i < NU; ++i)
                if (fu + 8 * i < units) f[r][i] = *reinterpret_cast<const bf16x8*>(src + 64 * i);
        }
    };
    auto store = [&](int at) __attribute__((always_inline)) {
#pragma unroll
        for (int r = 0; r < kTileRows; ++r)
#pragma unroll
            for (int i = 0; i < NU; ++i)
                if (fu + 8 * i < units) *reinterpret_cast<bf16x8*>(kt + at + tile_unit(fkey + kRowStep * r, ks, fu + 8 * i)) = f[r][i];
    };
    fetch(0);
    store(0);
    int now = 0;
    for (int it = 0; it < tiles; ++it, now = buffer - now) {
        const bool more = it + 1 < tiles, window_tile = it >= kept_tiles;
        const int j0 = first_key(it);
        if (more) fetch(it + 1);
        __syncthreads();  // this tile is written, and nobody reads the other buffer any more
        // (uniform per wave) does this wave see anything of the tile, and does it see all of it?
        const bool any = busy && (window_tile ? j0 <= own_hi && (j0 + kTileKeys - 1 > own_lo - L.window || j0 < keep) : true);
        const bool all = window_tile ? j0 + kTileKeys - 1 <= own_lo && j0 > own_hi - L.window : j0 + kTileKeys <= kept;
        if (any) {
            f32x4 sc[4][2];
#pragma unroll
            for (int x = 0; x < 4; ++x)
#pragma unroll
                for (int t = 0; t < 2; ++t) sc[x][t] = f32x4{0.f, 0.f, 0.f, 0.f};
            TAH_WAVE_PRIORITY(1);  // (a wave in a run of products goes before one in its softmax: the two then alternate)
#pragma unroll
            for (int s = 0; s < NQ; ++s) {
                if (kExact || s < nq) {
#pragma unroll
                    for (int x = 0; x < 4; ++x) {
                        const bf16x8 a = *reinterpret_cast<const bf16x8*>(kt + now + k_at + 16 * x * ks + 32 * s);
#pragma unroll
                        for (int t = 0; t < 2; ++t) sc[x][t] = mfma16(a, q[t][s], sc[x][t]);
                    }
                }
            }
            TAH_WAVE_PRIORITY(0);
            bf16x8 ph[2][2], pl[2][2];  // [pair of key tiles][query tile]
#pragma unroll
            for (int t = 0; t < 2; ++t) {
                if (!all) {
                    // kept tokens' tiles end at `kept` (what follows comes again with the window's tiles)
                    // (as distances from this lane's first key)
                    const int base = j0 + 4 * gq, lo = own[t] - L.window - base, hi = (window_tile ? own[t] : kept - 1) - base;
                    const int from = (window_tile ? keep : kept) - base, start = (window_tile ? j_lo : 0) - base;
#pragma unroll
                    for (int x = 0; x < 4; ++x)
#pragma unroll
                        for (int r = 0; r < 4; ++r) {
                            const int j = 16 * x + r;
                            const bool off = (j > hi) | ((j <= lo) & (j >= from)) | (j < start);
                            sc[x][t][r] = off ? kNegInf : sc[x][t][r];
                        }
                }
                // (maximum before the scale, which is positive; scale and difference are one multiply-add)
                float mx = score_max(sc[0][t][0], sc[0][t][1]);
#pragma unroll
                for (int e = 2; e < 16; ++e) mx = score_max(mx, sc[e / 4][t][e % 4]);
                // The weights are taken against a running reference, not the maximum itself: it moves only when a score of the wave
                // passes it by kSlack, so that most tiles leave the sums alone; weights stay below 2^kSlack.
                mx = fmaxf(m[t], groups_max(mx) * p.scale_log2);
                if (__ballot(mx > m[t] + kSlack) != 0) {
                    const float a = fast_exp2(m[t] - mx);
                    m[t] = mx;
#pragma unroll
                    for (int i = 0; i < NV; ++i)
#pragma unroll
                        for (int r = 0; r < 4; ++r) acc[i][t][r] *= a;
#pragma unroll
                    for (int r = 0; r < 4; ++r) l[t][r] *= a;
                }
#pragma unroll
                for (int x = 0; x < 2; ++x) {
                    float w[8];
#pragma unroll
                    for (int e = 0; e < 8; ++e) w[e] = fast_exp2(__builtin_fmaf(sc[2 * x + e / 4][t][e % 4], p.scale_log2, -m[t]));
                    split_bf16x8(w, ph[x][t], pl[x][t]);
                }
            }
            TAH_WAVE_PRIORITY(1);
#pragma unroll
            for (int t = 0; t < 2; ++t) {
                // the weights' sums, all keys of the tile at once, in every row of the result
#pragma unroll
                for (int x = 0; x < 2; ++x) {
                    l[t] = mfma16(ones, ph[x][t], l[t]);
                    l[t] = mfma16(ones, pl[x][t], l[t]);
                }
            }
#pragma unroll
            for (int i = 0; i < NV; ++i)
                if (kExact || i < nv) {
#pragma unroll
                    for (int x = 0; x < 2; ++x) {
                        const __bf16* at = kt + now + v_at + 32 * x * ks + 16 * i;
                        const bf16x8 a = join8(lds_read_tr16(reinterpret_cast<const unsigned char*>(at)),
                                               lds_read_tr16(reinterpret_cast<const unsigned char*>(at + 16 * ks)));
#pragma unroll
                        for (int t = 0; t < 2; ++t) acc[i][t] = mfma16(a, ph[x][t], acc[i][t]);
#pragma unroll
                        for (int t = 0; t < 2; ++t) acc[i][t] = mfma16(a, pl[x][t], acc[i][t]);
                    }
                }
            TAH_WAVE_PRIORITY(0);
        }
        if (more) store(buffer - now);
    }
#pragma unroll
    for (int t = 0; t < 2; ++t) {
        float inv = 1.0f / l[t][0];
        if (on[t]) {
            if (R.g_col >= 0) inv *= sigmoid_exact((float)proj[(int64_t)qrow[t] * R.proj_row_stride + R.g_col + head[t]]);
            __bf16* const out = static_cast<__bf16*>(p.c.out) + (int64_t)qrow[t] * p.c.out_rs + (int64_t)head[t] * L.value_dim + 4 * gq;
#pragma unroll
            for (int i = 0; i < NV; ++i)
                if (kExact || i < nv) {
                    bf16x4 y;
#pragma unroll
                    for (int e = 0; e < 4; ++e) y[e] = (__bf16)(acc[i][t][e] * inv);
                    *reinterpret_cast<bf16x4*>(out + 16 * i) = y;
                }
        }
    }
}

// ---- single tokens on the matrix cores ---------------------------------------------------------------------------
constexpr int kDecKeys = 32;  // keys a wave takes at a time

struct WindowDecode {
    tah_window_layer L;
    tah_window_rows R;
    __bf16 *out, *out_packed;
    int64_t out_rs;
    float* part;  // [rows][heads][splits][value_dim + 4]: sums, the maximum, the sum of weights; NULL with one split
    int32_t splits, keys_per_split, chunks;
    float scale_log2;
};

// grid (splits, kv_heads * chunks of 16 query heads, rows).  NQ, NV as above; NU: 16-byte units of a row per lane (at most; eight
// lanes to a row, four rows a lane); W: waves.  LDS: W tiles of 32 rows (later the waves' results), 16 queries, a rotated key.
template <int NQ, int NV, int NU, int W, bool kExact>
__global__ __launch_bounds__(W * kWave) void window_decode_kernel(const WindowDecode p) {
    HIP_DYNAMIC_SHARED(unsigned char, dec_lds)
    __shared__ float mx_[W][16], sum_[W][16];
    constexpr int kThreads = W * kWave;
    const tah_window_layer& L = p.L;
    const tah_window_rows& R = p.R;
    const int row = blockIdx.z, tid = threadIdx.x, lane = tid % kWave, wave = tid / kWave, c = lane % 16, gq = lane / 16;
    const int g = blockIdx.y / p.chunks, chunk = blockIdx.y % p.chunks, per = L.heads / L.kv_heads;
    const int h0 = g * per + 16 * chunk, nh = per - 16 * chunk < 16 ? per - 16 * chunk : 16;
    const int nq = kExact ? NQ : L.key_dim / 32, nv = kExact ? NV : L.value_dim / 16;
    const int ks = tile_stride(L.row), koff = L.row - L.key_dim, qs = L.key_dim + 8, units = L.row / 8;
    __bf16* const kt = reinterpret_cast<__bf16*>(dec_lds) + wave * kDecKeys * ks;
    __bf16* const qt = reinterpret_cast<__bf16*>(dec_lds) + W * kDecKeys * ks;
    __bf16* const kr = qt + 16 * qs;  // [rot_pad]: the new key's rotated part
    const int p0 = R.pos[row];
    int slot = R.slot[row];
    if (slot >= L.nslots) slot = -1;
    const bool live = slot >= 0 && p0 >= 0;
    const int pos = p0 < 0 ? 0 : p0;
    const __bf16* const proj = static_cast<const __bf16*>(R.proj) + (int64_t)row * R.proj_row_stride;
    const __bf16* const fresh = proj + R.k_col + g * L.row;
    __bf16* const cache = static_cast<__bf16*>(L.cache) + ((int64_t)(slot < 0 ? 0 : slot) * L.kv_heads + g) * (L.keep_first + L.ring) * L.row;
    int lo = pos - L.window + 1;
    lo = lo < 0 ? 0 : lo;
    const RingView view(L.keep_first, L.ring, lo);
    const int kept = L.keep_first < lo ? L.keep_first : lo, nk = live ? kept + pos - lo + 1 : 0;  // kept first tokens, then the window
    const int begin = blockIdx.x * p.keys_per_split;
    const int end = begin + p.keys_per_split < nk ? begin + p.keys_per_split : nk;
    const int fkey = lane / 8, fu = lane % 8;  // this lane's rows fkey + 8 r, and units fu, fu + 8, ... of them
    bf16x8 fa[4][NU], fb[4][NU];
    auto fetch = [&](int x0, bf16x8 (&f)[4][NU]) __attribute__((always_inline)) {
#pragma unroll
        for (int r = 0; r < 4; ++r) {
            int x = x0 + fkey + 8 * r;
            x = x < nk ? x : nk - 1;
            const __bf16* const src = (x == nk - 1 ? fresh : cache + view.row(x < kept ? x : lo + x - kept) * L.row) + 8 * fu;
#pragma unroll
            for (int i = 0; i < NU; ++i)
                if (fu + 8 * i < units) f[r][i] = *reinterpret_cast<const bf16x8*>(src + 64 * i);
        }
    };
    constexpr int kPass = W * kDecKeys, kAhead = NQ <= 4 ? 2 : 1;  // passes whose rows are under way at a time
    int x0 = begin + wave * kDecKeys;
    if (x0 < end) fetch(x0, fa);
    if (kAhead > 1 && x0 + kPass < end) fetch(x0 + kPass, fb);
    // queries (heads past the last one repeat it; nobody reads them) and the new key's rotated part
    const int half = L.rot_dim / 2, tpos = pos < R.table_rows ? pos : R.table_rows - 1, rot0 = L.key_dim - L.rot_pad;
    const float* const co = R.cos + (int64_t)tpos * half;
    const float* const si = R.sin + (int64_t)tpos * half;
    auto rotated = [&](bf16x8 v, int m0) __attribute__((always_inline)) {  // pairs m0 ... m0 + 3
#pragma unroll
        for (int i = 0; i < 4; ++i)
            if (m0 + i < half) {
                const float a = (float)v[2 * i], b = (float)v[2 * i + 1], cs = co[m0 + i], sn = si[m0 + i];
                v[2 * i] = (__bf16)(a * cs - b * sn);
                v[2 * i + 1] = (__bf16)(b * cs + a * sn);
            }
        return v;
    };
    const int uq = L.key_dim / 8;
    for (int u = tid; u < 16 * uq; u += kThreads) {
        const int h = u / uq, x = 8 * (u % uq);
        bf16x8 v = *reinterpret_cast<const bf16x8*>(proj + R.q_col + (h0 + (h < nh ? h : nh - 1)) * L.key_dim + x);
        if (x >= rot0) v = rotated(v, (x - rot0) / 2);
        *reinterpret_cast<bf16x8*>(qt + h * qs + x) = v;
    }
    for (int x = 8 * tid; x < L.rot_pad; x += 8 * kThreads)
        *reinterpret_cast<bf16x8*>(kr + x) = rotated(*reinterpret_cast<const bf16x8*>(fresh + L.rot_source + x), x / 2);
    __syncthreads();
    bf16x8 q[NQ];
#pragma unroll
    for (int s = 0; s < NQ; ++s)
        if (kExact || s < nq) q[s] = *reinterpret_cast<const bf16x8*>(qt + c * qs + 32 * s + 8 * gq);
    f32x4 acc[NV];
#pragma unroll
    for (int i = 0; i < NV; ++i) acc[i] = f32x4{0.f, 0.f, 0.f, 0.f};
    float m = kNoScore, l = 0.f;
    auto step = [&](bf16x8 (&f)[4][NU]) __attribute__((always_inline)) {
#pragma unroll
        for (int r = 0; r < 4; ++r) {
            const int key = fkey + 8 * r, x = x0 + key;
#pragma unroll
            for (int i = 0; i < NU; ++i)
                if (fu + 8 * i < units) {
                    const int at = 8 * (fu + 8 * i);
                    if (x >= nk - 1) {  // the new token: its rotated part, and its place in the cache
                        if (at >= L.row - L.rot_pad) f[r][i] = *reinterpret_cast<const bf16x8*>(kr + at - (L.row - L.rot_pad));
                        if (x == nk - 1 && chunk == 0) *reinterpret_cast<bf16x8*>(cache + view.row(pos) * L.row + at) = f[r][i];
                    }
                    *reinterpret_cast<bf16x8*>(kt + tile_unit(key, ks, fu + 8 * i)) = f[r][i];
                }
        }
        TAH_WAVE_LDS_SYNC();
        if (x0 + kAhead * kPass < end) fetch(x0 + kAhead * kPass, f);
        // register r of sc[x], lane (c, gq): key 16 x + 4 gq + r, head c
        f32x4 sc[2];
#pragma unroll
        for (int x = 0; x < 2; ++x) {
            sc[x] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
            for (int s = 0; s < NQ; ++s)
                if (kExact || s < nq)
                    sc[x] = mfma16(*reinterpret_cast<const bf16x8*>(kt + tile_unit(16 * x + c, ks, koff / 8 + 4 * s + gq)), q[s], sc[x]);
        }
        float mw = kNoScore;
#pragma unroll
        for (int x = 0; x < 2; ++x)
#pragma unroll
            for (int r = 0; r < 4; ++r) {
                sc[x][r] = x0 + 16 * x + 4 * gq + r < end ? sc[x][r] * p.scale_log2 : kNegInf;
                mw = fmaxf(mw, sc[x][r]);
            }
        const float mn = fmaxf(m, groups_max(mw)), a = fast_exp2(m - mn);
        m = mn;
        l *= a;
        bf16x8 ph, pl;
        float w[8];
#pragma unroll
        for (int e = 0; e < 8; ++e) {
            w[e] = fast_exp2(sc[e / 4][e % 4] - mn);
            l += w[e];
        }
        split_bf16x8(w, ph, pl);
#pragma unroll
        for (int i = 0; i < NV; ++i)
            if (kExact || i < nv) {
                const __bf16* const at = kt + tile_unit(4 * gq + c / 4, ks, 2 * i + c % 4 / 2) + 4 * (c % 2);
                const bf16x8 v = join8(lds_read_tr16(reinterpret_cast<const unsigned char*>(at)),
                                       lds_read_tr16(reinterpret_cast<const unsigned char*>(at + 16 * ks)));
#pragma unroll
                for (int r = 0; r < 4; ++r) acc[i][r] *= a;
                acc[i] = mfma16(v, ph, acc[i]);
                acc[i] = mfma16(v, pl, acc[i]);
            }
        TAH_WAVE_LDS_SYNC();  // the tile is read before it is written again
        x0 += kPass;
    };
    while (x0 < end) {
        step(fa);
        if (kAhead > 1 && x0 < end) step(fb);
    }
    // the waves' results meet in LDS: [wave][head][value_dim + 4] over the tiles
    l = groups_sum(l);
    __syncthreads();
    float* const res = reinterpret_cast<float*>(dec_lds);
    const int vs = L.value_dim + 4;
    if (gq == 0) {
        mx_[wave][c] = m;
        sum_[wave][c] = l;
    }
    if (c < nh) {
#pragma unroll
        for (int i = 0; i < NV; ++i)
            if (kExact || i < nv) *reinterpret_cast<f32x4*>(res + (wave * nh + c) * vs + 16 * i + 4 * gq) = acc[i];
    }
    __syncthreads();
    const int upv = L.value_dim / 8;
    for (int u = tid; u < nh * upv; u += kThreads) {
        const int h = u / upv, x = 8 * (u % upv);
        float mm = kNoScore, ll = 0.f, y[8] = {0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int w = 0; w < W; ++w) mm = fmaxf(mm, mx_[w][h]);
#pragma unroll
        for (int w = 0; w < W; ++w) {
            const float a = fast_exp2(mx_[w][h] - mm);  // (a wave that saw nothing has no weights and zeros)
            float v[8];
            load8(res + (w * nh + h) * vs + x, v);
            ll += sum_[w][h] * a;
#pragma unroll
            for (int e = 0; e < 8; ++e) y[e] += v[e] * a;
        }
        if (p.part) {
            float* const o = p.part + (((int64_t)row * L.heads + h0 + h) * p.splits + blockIdx.x) * vs;
            store8(o + x, y);
            if (x == 0) {
                o[L.value_dim] = mm;
                o[L.value_dim + 1] = ll;
            }
            continue;
        }
        float inv = ll > 0.f ? 1.0f / ll : 0.f;
        if (R.g_col >= 0) inv *= sigmoid_exact((float)proj[R.g_col + h0 + h]);
#pragma unroll
        for (int e = 0; e < 8; ++e) y[e] *= inv;
        const int col = (h0 + h) * L.value_dim + x;
        if (p.out) store8(p.out + row * p.out_rs + col, y);
        if (p.out_packed) reinterpret_cast<bf16x8*>(p.out_packed)[rows_form_unit(row, col)] = to_bf16x8(y);
    }
}

// grid (heads, rows); eight value columns per thread, whose parts are all asked for before the first is used
__global__ __launch_bounds__(kWave) void window_merge_kernel(const WindowDecode p) {
    const int h = blockIdx.x, row = blockIdx.y, vs = p.L.value_dim + 4;
    const __bf16* const proj = static_cast<const __bf16*>(p.R.proj) + (int64_t)row * p.R.proj_row_stride;
    const float* const base = p.part + ((int64_t)row * p.L.heads + h) * p.splits * vs;
    for (int x = 8 * threadIdx.x; x < p.L.value_dim; x += 8 * kWave) {
        float m = kNoScore, l = 0.f, y[8] = {0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f};
        for (int s0 = 0; s0 < p.splits; s0 += 4) {
            float v[4][8], vm[4], vl[4];
#pragma unroll
            for (int i = 0; i < 4; ++i) {
                const float* const at = base + (int64_t)(s0 + i < p.splits ? s0 + i : p.splits - 1) * vs;
                load8(at + x, v[i]);
                vm[i] = at[p.L.value_dim];
                vl[i] = at[p.L.value_dim + 1];
            }
#pragma unroll
            for (int i = 0; i < 4; ++i) {
                if (s0 + i >= p.splits || !(vl[i] > 0.f)) continue;
                const float mn = fmaxf(m, vm[i]), a = fast_exp2(m - mn), b = fast_exp2(vm[i] - mn);
                m = mn;
                l = l * a + vl[i] * b;
#pragma unroll
                for (int e = 0; e < 8; ++e) y[e] = y[e] * a + v[i][e] * b;
            }
        }
        float inv = l > 0.f ? 1.0f / l : 0.f;
        if (p.R.g_col >= 0) inv *= sigmoid_exact((float)proj[p.R.g_col + h]);
#pragma unroll
        for (int e = 0; e < 8; ++e) y[e] *= inv;
        const int col = h * p.L.value_dim + x;
        if (p.out) store8(p.out + row * p.out_rs + col, y);
        if (p.out_packed) reinterpret_cast<bf16x8*>(p.out_packed)[rows_form_unit(row, col)] = to_bf16x8(y);
    }
}

int check_layer(const tah_window_layer* L) {
    if (!L) return TAH_E_NULL;
    if (L->heads <= 0 || L->kv_heads <= 0 || L->heads % L->kv_heads != 0 || L->heads > 65535 || L->key_dim <= 0 || L->key_dim % 32 != 0 ||
        L->value_dim <= 0 || L->value_dim % 32 != 0 || L->row % 8 != 0 || L->row < L->key_dim || L->row < L->value_dim ||
        L->row > L->key_dim + L->value_dim || (L->row - L->key_dim) % 16 != 0 || L->rot_dim < 0 || L->rot_dim % 2 != 0 ||
        L->rot_pad % 16 != 0 || L->rot_pad < L->rot_dim || L->rot_pad > L->key_dim || L->rot_source < 0 || L->rot_source % 8 != 0 || L->rot_source + L->rot_pad > L->row || L->keep_first < 0 ||
        L->ring <= 0 || (int64_t)(L->keep_first + (int64_t)L->ring) * L->row >= (1 << 30) || L->window <= 0 || L->window > L->ring ||
        L->nslots <= 0 || (L->dtype != TAH_DT_BF16 && L->dtype != TAH_DT_F32))
        return TAH_E_SHAPE;
    if (L->key_dim > 8192 || L->value_dim > kWinThreads * kRowValues) return TAH_E_SHAPE;
    if (!L->cache) return TAH_E_NULL;
    return aligned_16(L->cache) ? TAH_OK : TAH_E_ALIGN;
}
int check_rows(const tah_window_layer* L, const tah_window_rows* R) {
    if (!R) return TAH_E_NULL;
    if (R->rows < 0 || R->q_col < 0 || R->q_col % 8 != 0 || R->k_col < 0 || R->k_col % 8 != 0 || R->proj_row_stride % 8 != 0 || R->table_rows <= 0)
        return TAH_E_SHAPE;
    if (R->proj_row_stride < R->q_col + (int64_t)L->heads * L->key_dim || R->proj_row_stride < R->k_col + (int64_t)L->kv_heads * L->row ||
        (R->g_col >= 0 && R->proj_row_stride < (int64_t)R->g_col + L->heads))
        return TAH_E_SHAPE;
    if (R->rows == 0) return TAH_OK;
    if (!R->proj || !R->pos || (L->rot_dim > 0 && (!R->cos || !R->sin))) return TAH_E_NULL;
    return aligned_16(R->proj) ? TAH_OK : TAH_E_ALIGN;
}
int check_portions(const tah_portions* p, const tah_window_rows* R) {
    if (!p) return TAH_E_NULL;
    if (p->nseq < 0 || p->rows != R->rows) return TAH_E_SHAPE;
    if (p->nseq > 0 && p->rows > 0 && (!p->cu || !p->slot || !p->pos0 || !p->row_seq)) return TAH_E_NULL;
    return TAH_OK;
}

void launch_rows(const WindowCall& c, hipStream_t st) {
    const size_t lds = (size_t)c.L.key_dim * sizeof(float);
    if (c.L.dtype == TAH_DT_BF16) hipLaunchKernelGGL((window_rows_kernel<__bf16>), dim3(c.R.rows, c.L.heads), dim3(kWinThreads), lds, st, c);
    else hipLaunchKernelGGL((window_rows_kernel<float>), dim3(c.R.rows, c.L.heads), dim3(kWinThreads), lds, st, c);
}
void launch_prep(const tah_window_layer& L, const tah_window_rows& R, hipStream_t st) {
    if (L.dtype == TAH_DT_BF16) hipLaunchKernelGGL((window_prep_kernel<__bf16>), dim3(R.rows), dim3(kWinThreads), 0, st, L, R);
    else hipLaunchKernelGGL((window_prep_kernel<float>), dim3(R.rows), dim3(kWinThreads), 0, st, L, R);
}

// ---- sizes the matrix kernels take: keys and values up to 256 per head
bool on_tiles(const tah_window_layer* L) {
    return L->dtype == TAH_DT_BF16 && L->key_dim <= 256 && L->value_dim <= 256 && L->scale > 0.f;
}

template <int NQ, int NV, int NU, bool kExact>
int launch_tile(WindowTile t, hipStream_t st) {
    const size_t lds = (size_t)2 * kTileKeys * tile_stride(t.c.L.row) * 2;
    const void* const f = reinterpret_cast<const void*>(&window_tile_kernel<NQ, NV, NU, kExact>);
    if (lds > 65536 && hipFuncSetAttribute(f, hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds) != hipSuccess) return TAH_E_LAUNCH;
    const int per = t.c.L.heads / t.c.L.kv_heads;
    t.chunks = (per + kTileQueries - 1) / kTileQueries;
    t.heads_per_tile = (per + t.chunks - 1) / t.chunks;
    t.slots = t.c.P.rows / (16 * (kTileQueries / t.heads_per_tile)) + t.c.P.nseq;
    const int64_t items = (int64_t)t.slots * t.c.L.kv_heads * t.chunks;
    if (items > (1 << 28)) return TAH_E_SHAPE;
    t.per_xcd = (int)((items + 7) / 8);
    hipLaunchKernelGGL((window_tile_kernel<NQ, NV, NU, kExact>), dim3((unsigned)(8 * t.per_xcd)), dim3(kTileThreads), lds, st, t);
    return launch_status();
}

// how a decode call splits its keys: enough workgroups for the chip, and work for every wave of one
constexpr int kDecodeGroups = 256;
int decode_waves(int row) { return row <= 256 ? 8 : 4; }
void decode_split(const tah_window_layer& L, int rows, int& splits, int& keys_per_split) {
    const int pass = kDecKeys * decode_waves(L.row), keys = L.keep_first + L.window;
    const int most = (keys + pass - 1) / pass, groups = rows * L.kv_heads * ((L.heads / L.kv_heads + 15) / 16);
    int want = groups > 0 ? (kDecodeGroups + groups - 1) / groups : 1;
    want = want < 1 ? 1 : (want > most ? most : want);
    const int tiles = (keys + kDecKeys - 1) / kDecKeys;
    keys_per_split = (tiles + want - 1) / want * kDecKeys;
    splits = (keys + keys_per_split - 1) / keys_per_split;
}

template <int NQ, int NV, int NU, int W, bool kExact>
int launch_decode(const WindowDecode& d, hipStream_t st) {
    const size_t tiles = (size_t)W * kDecKeys * tile_stride(d.L.row) * 2, tail = ((size_t)16 * (d.L.key_dim + 8) + d.L.rot_pad) * 2;
    const size_t results = (size_t)W * 16 * (d.L.value_dim + 4) * sizeof(float);
    const size_t lds = tiles + tail > results ? tiles + tail : results;
    const void* const f = reinterpret_cast<const void*>(&window_decode_kernel<NQ, NV, NU, W, kExact>);
    if (lds > 65536 && hipFuncSetAttribute(f, hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds) != hipSuccess) return TAH_E_LAUNCH;
    hipLaunchKernelGGL((window_decode_kernel<NQ, NV, NU, W, kExact>), dim3(d.splits, d.L.kv_heads * d.chunks, d.R.rows), dim3(W * kWave), lds, st, d);
    return launch_status();
}

}  // namespace
}  // namespace tah

extern "C" int tah_window_prep(const tah_window_layer* L, const tah_window_rows* R, tah_stream_t stream) {
    using namespace tah;
    if (const int rc = check_layer(L)) return rc;
    if (const int rc = check_rows(L, R)) return rc;
    if (R->rows == 0) return TAH_OK;
    launch_prep(*L, *R, static_cast<hipStream_t>(stream));
    return launch_status();
}

extern "C" int tah_window_attend(const tah_window_layer* L, const tah_portions* P, const tah_window_rows* R, void* out, int64_t out_rs,
                                 tah_stream_t stream) {
    using namespace tah;
    if (const int rc = check_layer(L)) return rc;
    if (const int rc = check_rows(L, R)) return rc;
    if (const int rc = check_portions(P, R)) return rc;
    if (out_rs % 8 != 0 || out_rs < (int64_t)L->heads * L->value_dim) return TAH_E_SHAPE;
    if (R->rows == 0 || P->nseq == 0) return TAH_OK;
    if (!out) return TAH_E_NULL;
    if (!aligned_16(out)) return TAH_E_ALIGN;
    hipStream_t st = static_cast<hipStream_t>(stream);
    const WindowCall c{*L, *R, *P, out, nullptr, out_rs};
    if (on_tiles(L)) {
        WindowTile t{};
        t.c = c;
        t.scale_log2 = L->scale * kLog2e;
        // (units per thread: row / 64, rounded up; rows are at most key_dim + value_dim elements)
        if (L->key_dim == 128 && L->value_dim == 128 && L->row <= 192) return launch_tile<4, 8, 3, true>(t, st);
        if (L->key_dim <= 64 && L->value_dim <= 64) return launch_tile<2, 4, 2, false>(t, st);
        if (L->key_dim <= 128 && L->value_dim <= 128) return launch_tile<4, 8, 4, false>(t, st);
        return launch_tile<8, 16, 8, false>(t, st);
    }
    launch_rows(c, st);
    return launch_status();
}

extern "C" int tah_window_append(const tah_window_layer* L, const tah_portions* P, const tah_window_rows* R, tah_stream_t stream) {
    using namespace tah;
    if (const int rc = check_layer(L)) return rc;
    if (const int rc = check_rows(L, R)) return rc;
    if (const int rc = check_portions(P, R)) return rc;
    if (R->rows == 0 || P->nseq == 0) return TAH_OK;
    hipStream_t st = static_cast<hipStream_t>(stream);
    const dim3 grid((R->rows + kWinWaves - 1) / kWinWaves);
    if (L->dtype == TAH_DT_BF16) hipLaunchKernelGGL((window_append_kernel<__bf16>), grid, dim3(kWinThreads), 0, st, *L, *P, *R);
    else hipLaunchKernelGGL((window_append_kernel<float>), grid, dim3(kWinThreads), 0, st, *L, *P, *R);
    return launch_status();
}

extern "C" size_t tah_window_decode_workspace(const tah_window_layer* L, int32_t rows) {
    if (tah::check_layer(L) != TAH_OK || rows <= 0 || !tah::on_tiles(L)) return 0;
    size_t most = 0;
    for (int r = 1; r <= rows; ++r) {  // enough for fewer rows too
        int splits, keys;
        tah::decode_split(*L, r, splits, keys);
        const size_t n = splits > 1 ? (size_t)r * L->heads * splits * (L->value_dim + 4) * sizeof(float) : 0;
        most = n > most ? n : most;
    }
    return most;
}

extern "C" int tah_window_decode(const tah_window_layer* L, const tah_window_rows* R, void* out, int64_t out_rs, void* out_packed, void* workspace,
                                 size_t workspace_bytes, tah_stream_t stream) {
    using namespace tah;
    if (const int rc = check_layer(L)) return rc;
    if (const int rc = check_rows(L, R)) return rc;
    if ((out && (out_rs % 8 != 0 || out_rs < (int64_t)L->heads * L->value_dim)) || (out_packed && (R->rows > 32 || L->dtype != TAH_DT_BF16)) ||
        R->rows > 65535)
        return TAH_E_SHAPE;
    if (R->rows == 0) return TAH_OK;
    if (!R->slot || (!out && !out_packed)) return TAH_E_NULL;
    if (!aligned_16(out) || !aligned_16(out_packed)) return TAH_E_ALIGN;
    hipStream_t st = static_cast<hipStream_t>(stream);
    if (!on_tiles(L)) {
        launch_prep(*L, *R, st);
        launch_rows(WindowCall{*L, *R, tah_portions{}, out, out_packed, out_rs}, st);
        return launch_status();
    }
    WindowDecode d{};
    d.L = *L; d.R = *R;
    d.out = static_cast<__bf16*>(out); d.out_packed = static_cast<__bf16*>(out_packed); d.out_rs = out_rs;
    d.scale_log2 = L->scale * kLog2e;
    d.chunks = (L->heads / L->kv_heads + 15) / 16;
    decode_split(*L, R->rows, d.splits, d.keys_per_split);
    if (d.splits > 1) {
        if (!workspace || !aligned_16(workspace) || workspace_bytes < (size_t)R->rows * L->heads * d.splits * (L->value_dim + 4) * sizeof(float))
            return TAH_E_WORKSPACE;
        d.part = static_cast<float*>(workspace);
    }
    // (units per lane and row: row / 64, rounded up)
    int rc;
    if (L->key_dim == 128 && L->value_dim == 128 && L->row <= 192) rc = launch_decode<4, 8, 3, 8, true>(d, st);
    else if (L->key_dim <= 64 && L->value_dim <= 64) rc = launch_decode<2, 4, 2, 8, false>(d, st);
    else if (L->row <= 256) rc = launch_decode<8, 16, 4, 8, false>(d, st);
    else rc = launch_decode<8, 16, 8, 4, false>(d, st);
    if (rc != TAH_OK || d.splits == 1) return rc;
    hipLaunchKernelGGL(window_merge_kernel, dim3(L->heads, R->rows), dim3(kWave), 0, st, d);
    return launch_status();
}
