// Sliding-window latent attention, gfx950.  A token's keys and values of all heads are linear in one latent c [rank];
// what is cached is c and a rotated key part shared by the heads, one row per token, in a ring per sequence that is
// as long as the widest window that reads it.
//
//  * latent_prep_kernel: projections of a step's or a portion's rows -> normed latents and rotated key part (into the
//    ring, or packed for tah_latent_context), rotated query part, and the unrotated query part in the operand order of
//    the per-head products.
//  * latent_context_kernel / latent_append_kernel: the rows a batch of portions can see, packed (old ones from the
//    ring, new ones from the portion), then the new rows into the ring.
//  * attend_tile_kernel (bf16): portions.  256 query rows of one head per workgroup (32 per wave) against 64 keys at a time, on the
//    matrix cores: S^T = K Q^T, so that a query's scores sit in one lane column and the softmax needs two shuffles, and
//    O^T = V^T P^T with V^T read from the row-major tile by transpose reads.  Keys outside the window are not visited.
//  * latent_decode_kernel / latent_merge_kernel (bf16): single tokens.  All heads (sixteen at a time) of one row share a
//    pass over the ring, which is both keys and values; the window is split over workgroups, and the parts are merged.
//  * attend_rows_kernel: one workgroup per (query, head), any sizes, either element type (the float32 form).
//
// Scores, weights and sums are float32.  Where a weight enters a bf16 matrix product it goes in as two bf16 terms
// (its rounding and what the rounding left), so that it keeps sixteen bits.
#include <hip/hip_runtime.h>

#include "mixer_device.h"

namespace tah {
namespace {

constexpr int kLatThreads = 256;
constexpr int kLatWaves = kLatThreads / kWave;

template <class E>
__global__ __launch_bounds__(kLatThreads) void latent_prep_kernel(const tah_latent_layer L, const tah_latent_prep_args p) {
    __shared__ float red[kLatWaves];
    const int row = blockIdx.x, tid = threadIdx.x;
    E* const pr = static_cast<E*>(p.proj) + (int64_t)row * p.proj_row_stride;
    int pos = p.pos[row];
    const int slot = p.slot ? p.slot[row] : -1;
    const bool live = pos >= 0;
    pos = pos < 0 ? 0 : (pos >= p.table_rows ? p.table_rows - 1 : pos);
    const int half = L.rot_dim / 2;
    const float* const co = p.cos + (int64_t)pos * half;
    const float* const si = p.sin + (int64_t)pos * half;
    const int lp = L.rank_pad + L.rot_pad, hq = L.dim_pad + L.rot_pad;
    if (p.dkv_col >= 0) {
        const E* const d = pr + p.dkv_col;
        float ss = 0.f;
        for (int i = tid; i < L.rank; i += kLatThreads) ss += (float)d[i] * (float)d[i];
        ss = block_sum<kLatWaves>(ss, red);
        const float r = 1.0f / sqrtf(ss / (float)L.rank + p.eps);
        E* const to_rows = p.rows_out ? static_cast<E*>(p.rows_out) + (int64_t)row * lp : nullptr;
        E* const to_ring = (live && slot >= 0 && slot < L.nslots)
                               ? static_cast<E*>(L.ring) + ((int64_t)slot * L.capacity + p.pos[row] % L.capacity) * lp : nullptr;
        for (int i = tid; i < lp; i += kLatThreads) {
            float y = 0.f;
            if (i < L.rank) y = (float)d[i] * r * p.norm[i];
            else if (i >= L.rank_pad && i < L.rank_pad + L.rot_dim) {
                const int j = i - L.rank_pad, m = j < half ? j : j - half;
                const float u = (float)d[L.rank + m], v = (float)d[L.rank + half + m];
                y = j < half ? u * co[m] - v * si[m] : v * co[m] + u * si[m];
            }
            if (to_rows) to_rows[i] = (E)y;
            if (to_ring) to_ring[i] = (E)y;
        }
    }
    for (int i = tid; i < L.heads * half; i += kLatThreads) {
        const int h = i / half, m = i % half;
        E* const q = pr + p.q_col + h * hq + L.dim_pad;
        const float u = (float)q[m], v = (float)q[half + m];
        q[m] = (E)(u * co[m] - v * si[m]);
        q[half + m] = (E)(v * co[m] + u * si[m]);
    }
    if (p.q_packed || p.q_rows) {
        for (int i = 8 * tid; i < L.heads * L.dim_pad; i += 8 * kLatThreads) {
            const int h = i / L.dim_pad, c = i % L.dim_pad;
            float v[8];
            load8(pr + p.q_col + h * hq + c, v);
            if (p.q_packed) static_cast<bf16x8*>(p.q_packed)[(int64_t)h * 4 * L.dim_pad + rows_form_unit(row, c)] = to_bf16x8(v);
            if (p.q_rows) store8(static_cast<E*>(p.q_rows) + ((int64_t)h * p.rows + row) * L.dim_pad + c, v);
        }
    }
}

// one wave per context row; U: 16-byte units per row
template <class E>
__global__ __launch_bounds__(kLatThreads) void latent_context_kernel(const tah_latent_layer L, const tah_portions P, const int32_t* cu_k, int ctx_rows,
                                                                     const E* new_rows, E* ctx) {
    const int lane = threadIdx.x % kWave, row = blockIdx.x * kLatWaves + threadIdx.x / kWave;
    if (row >= ctx_rows) return;
    int lo = 0, hi = P.nseq - 1;  // the last sequence whose context starts at or before this row and is not empty
    while (lo < hi) {
        const int mid = (lo + hi + 1) / 2;
        if (cu_k[mid] <= row) lo = mid; else hi = mid - 1;
    }
    const int b = lo, n = P.cu[b + 1] - P.cu[b], lk = cu_k[b + 1] - cu_k[b];
    const int pos = P.pos0[b] + n - lk + row - cu_k[b], lp = L.rank_pad + L.rot_pad;
    const int slot = P.slot[b];
    const E* src = pos >= P.pos0[b] ? new_rows + (int64_t)(P.cu[b] + pos - P.pos0[b]) * lp
                                    : static_cast<const E*>(L.ring) + ((int64_t)(slot < 0 ? 0 : slot) * L.capacity + pos % L.capacity) * lp;
    for (int c = 8 * lane; c < lp; c += 8 * kWave) {
        float v[8];
        load8(src + c, v);
        store8(ctx + (int64_t)row * lp + c, v);
    }
}

template <class E>
__global__ __launch_bounds__(kLatThreads) void latent_append_kernel(const tah_latent_layer L, const tah_portions P, const E* new_rows) {
    const int lane = threadIdx.x % kWave, row = blockIdx.x * kLatWaves + threadIdx.x / kWave;
    if (row >= P.rows) return;
    const int b = P.row_seq[row], slot = P.slot[b];
    if (slot < 0 || slot >= L.nslots || P.cu[b + 1] - row > L.capacity) return;  // (overwritten by a later row of the portion)
    const int pos = P.pos0[b] + row - P.cu[b], lp = L.rank_pad + L.rot_pad;
    E* const dst = static_cast<E*>(L.ring) + ((int64_t)slot * L.capacity + pos % L.capacity) * lp;
    for (int c = 8 * lane; c < lp; c += 8 * kWave) {
        float v[8];
        load8(new_rows + (int64_t)row * lp + c, v);
        store8(dst + c, v);
    }
}

// ---- any sizes, either element type: one workgroup per (query row, head) ----------------------------------------
struct AttendRows {
    // query: n1 elements at q1, n2 at q2; keys in two parts likewise; values nv elements
    const void *q1, *q2, *k1, *k2, *v;
    int64_t q1_rs, q1_hs, q2_rs, q2_hs, k1_rs, k1_hs, k2_rs, v_rs, v_hs;
    int32_t n1, n2, nv;
    // where a row's keys are: a ring (slot, pos given), or the packed context of its portion
    const int32_t *slot, *pos;
    const int32_t *cu, *cu_k, *pos0, *row_seq;
    int32_t capacity, nslots, window, rows;
    float scale;
    void* out;           // [.., nv] at row * out_rs + head * out_hs
    int64_t out_rs, out_hs;
    void* out_packed;    // rows form per head, 32 * nv elements each
};

constexpr int kAttKeys = 64;   // keys per pass
constexpr int kAttValues = 4;  // value elements per thread: nv <= 1024

template <class E>
__global__ __launch_bounds__(kLatThreads) void attend_rows_kernel(const AttendRows p) {
    HIP_DYNAMIC_SHARED(float, qs)   // [n1 + n2]
    __shared__ float sc[kAttKeys];
    const int row = blockIdx.x, h = blockIdx.y, tid = threadIdx.x, lane = tid % kWave, wave = tid / kWave;
    int64_t base;  // key row of position 0 (packed context)
    int pos, slot = 0;
    if (p.slot) {
        pos = p.pos[row];
        slot = p.slot[row];
        if (slot >= p.nslots) slot = -1;
        base = (int64_t)(slot < 0 ? 0 : slot) * p.capacity;
    } else {
        const int b = p.row_seq[row], n = p.cu[b + 1] - p.cu[b];
        pos = p.pos0[b] + row - p.cu[b];
        base = (int64_t)p.cu_k[b] - (p.pos0[b] + n - (p.cu_k[b + 1] - p.cu_k[b]));
    }
    const bool live = slot >= 0 && pos >= 0;
    auto key_row = [&](int j) __attribute__((always_inline)) { return p.slot ? base + j % p.capacity : base + j; };
    const E* q1 = static_cast<const E*>(p.q1) + row * p.q1_rs + h * p.q1_hs;
    const E* q2 = static_cast<const E*>(p.q2) + row * p.q2_rs + h * p.q2_hs;
    for (int i = tid; i < p.n1 + p.n2; i += kLatThreads) qs[i] = (float)(i < p.n1 ? q1[i] : q2[i - p.n1]);
    __syncthreads();
    float acc[kAttValues], m = kNegInf, l = 0.f;
#pragma unroll
    for (int e = 0; e < kAttValues; ++e) acc[e] = 0.f;
    int lo = pos - p.window + 1;
    lo = lo < 0 ? 0 : lo;
    for (int j0 = lo; live && j0 <= pos; j0 += kAttKeys) {
        for (int x = wave; x < kAttKeys; x += kLatWaves) {
            const int j = j0 + x;
            float s = 0.f;
            if (j <= pos) {
                const int64_t kr = key_row(j);
                const E* k1 = static_cast<const E*>(p.k1) + kr * p.k1_rs + h * p.k1_hs;
                const E* k2 = static_cast<const E*>(p.k2) + kr * p.k2_rs;
                for (int i = lane; i < p.n1; i += kWave) s += qs[i] * (float)k1[i];
                for (int i = lane; i < p.n2; i += kWave) s += qs[p.n1 + i] * (float)k2[i];
            }
            s = wave_sum(s);
            if (lane == 0) sc[x] = j <= pos ? s * p.scale : kNegInf;
        }
        __syncthreads();
        const float mn = fmaxf(m, wave_max(sc[lane]));
        const float a = expf(m - mn);  // (exp(-inf) = 0 the first time)
        m = mn;
        l = l * a + wave_sum(expf(sc[lane] - m));
#pragma unroll
        for (int e = 0; e < kAttValues; ++e) acc[e] *= a;
        const int nk = pos - j0 + 1 < kAttKeys ? pos - j0 + 1 : kAttKeys;
        for (int x = 0; x < nk; ++x) {
            const float w = expf(sc[x] - m);
            const E* v = static_cast<const E*>(p.v) + key_row(j0 + x) * p.v_rs + h * p.v_hs;
#pragma unroll
            for (int e = 0; e < kAttValues; ++e) {
                const int i = tid + e * kLatThreads;
                if (i < p.nv) acc[e] += w * (float)v[i];
            }
        }
        __syncthreads();
    }
#pragma unroll
    for (int e = 0; e < kAttValues; ++e) {
        const int i = tid + e * kLatThreads;
        if (i >= p.nv) continue;
        const float y = live ? acc[e] / l : 0.f;
        if (p.out) static_cast<E*>(p.out)[row * p.out_rs + h * p.out_hs + i] = (E)y;
        if (p.out_packed) static_cast<__bf16*>(p.out_packed)[(int64_t)h * 32 * p.nv + rows_form_elem(row, i)] = (__bf16)y;
    }
}

// ---- bf16 on the matrix cores ------------------------------------------------------------------------------------
constexpr int kTileKeys = 64;

struct AttendTile {
    const __bf16 *q, *k, *v, *ctx;  // q: head base [dim_pad | rot_pad]; ctx: rotated key part of context row 0
    int64_t q_rs, k_rs, v_rs, ctx_rs;
    __bf16* out;
    int64_t out_rs;
    const int32_t *cu, *cu_k;
    int32_t nseq, dim_pad, rot_pad, vdim_pad, window, heads, slots;
    float scale_log2;
};

// NQ: 32-wide steps of a query row (at most), NV: 16-wide tiles of a value row (at most; kExact: just so many, and no
// branch stands between a tile's products), W: waves, 32 query rows each.
template <int NQ, int NV, int W, bool kExact>
__global__ __launch_bounds__(W * kWave) void attend_tile_kernel(const AttendTile p) {
    constexpr int kTileRows = 32 * W, kTileThreads = W * kWave;
    HIP_DYNAMIC_SHARED(unsigned char, tile_lds)
    // (workgroups go to the XCDs round robin: where the heads divide among them, a head's tiles share an XCD and its L2)
    int tile, b = 0, row0 = 0, row_end = 0, h;
    if (p.heads % 8 == 0) {
        tile = blockIdx.x / 8 % p.slots;
        h = blockIdx.x / 8 / p.slots * 8 + blockIdx.x % 8;
    } else {
        tile = blockIdx.x % p.slots;
        h = blockIdx.x / p.slots;
    }
    if (!find_tile(p.cu, p.nseq, kTileRows, tile, b, row0, row_end)) return;
    const int tid = threadIdx.x, lane = tid % kWave, wave = tid / kWave, c = lane % 16, g = lane / 16;
    const int dq = p.dim_pad + p.rot_pad, nq = kExact ? NQ : dq / 32, nv = kExact ? NV : p.vdim_pad / 16;
    const int ks = dq + 8, vs = p.vdim_pad + 16;  // row strides in LDS: what a read takes from several rows lies in different banks
    __bf16* const kt = reinterpret_cast<__bf16*>(tile_lds);
    __bf16* const vt = kt + kTileKeys * ks;
    const int buffer = kTileKeys * (ks + vs);  // two of them: the next tile is written while this one is read
    const int first = p.cu[b], n = p.cu[b + 1] - first, k0 = p.cu_k[b], lk = p.cu_k[b + 1] - k0;
    // a query row's own key, as a context row of its sequence: row - first + lk - n
    const int shift = lk - n - first;
    const int wrow = row0 + 32 * wave;
    bf16x8 q[2][NQ];
    int own[2];
#pragma unroll
    for (int t = 0; t < 2; ++t) {
        int r = wrow + 16 * t + c;
        r = r < row_end ? r : row_end - 1;  // rows past the end repeat the last one and are not stored
        own[t] = r + shift;
#pragma unroll
        for (int s = 0; s < NQ; ++s)
            if (kExact || s < nq) q[t][s] = *reinterpret_cast<const bf16x8*>(p.q + (int64_t)r * p.q_rs + (int64_t)h * dq + 32 * s + 8 * g);
    }
    const int own_lo = (wrow < row_end ? wrow : row_end - 1) + shift;
    const int own_hi = (wrow + 31 < row_end ? wrow + 31 : row_end - 1) + shift;
    int j_lo = row0 + shift - p.window + 1;
    j_lo = j_lo < 0 ? 0 : j_lo;
    const int j_hi = row_end - 1 + shift;
    f32x4 acc[NV][2];
    float m[2] = {kNoScore, kNoScore}, l[2] = {0.f, 0.f};
#pragma unroll
    for (int i = 0; i < NV; ++i)
#pragma unroll
        for (int t = 0; t < 2; ++t) acc[i][t] = f32x4{0.f, 0.f, 0.f, 0.f};
    // a thread's sixteen-byte units of a tile, of the keys and of the values: where they come from and go to
    constexpr int UK = (kTileKeys * NQ * 4 + kTileThreads - 1) / kTileThreads, UV = (kTileKeys * NV * 2 + kTileThreads - 1) / kTileThreads;
    const int uk = dq / 8, ukn = p.dim_pad / 8, uv = p.vdim_pad / 8;
    const __bf16 *gk[UK], *gv[UV];
    int kkey[UK], vkey[UV], kdst[UK], vdst[UV];
    int64_t krs[UK];
    bf16x8 fk[UK], fv[UV];
#pragma unroll
    for (int i = 0; i < UK; ++i) {
        const int u = tid + kTileThreads * i, key = u / uk, x = u % uk;
        kkey[i] = u < kTileKeys * uk ? key : -1;
        kdst[i] = key * ks + 8 * x;
        gk[i] = x < ukn ? p.k + (int64_t)k0 * p.k_rs + (int64_t)h * p.dim_pad + 8 * x : p.ctx + (int64_t)k0 * p.ctx_rs + 8 * (x - ukn);
        krs[i] = x < ukn ? p.k_rs : p.ctx_rs;
    }
#pragma unroll
    for (int i = 0; i < UV; ++i) {
        const int u = tid + kTileThreads * i, key = u / uv, x = u % uv;
        vkey[i] = u < kTileKeys * uv ? key : -1;
        vdst[i] = key * vs + 8 * x;
        gv[i] = p.v + (int64_t)k0 * p.v_rs + (int64_t)h * p.vdim_pad + 8 * x;
    }
    auto fetch = [&](int j0) __attribute__((always_inline)) {
#pragma unroll
        for (int i = 0; i < UK; ++i) {
            const int j = j0 + kkey[i];
            if (kkey[i] >= 0) fk[i] = *reinterpret_cast<const bf16x8*>(gk[i] + (j < lk ? j : lk - 1) * krs[i]);
        }
#pragma unroll
        for (int i = 0; i < UV; ++i) {
            const int j = j0 + vkey[i];
            if (vkey[i] >= 0) fv[i] = *reinterpret_cast<const bf16x8*>(gv[i] + (j < lk ? j : lk - 1) * p.v_rs);
        }
    };
    auto store = [&](int at) __attribute__((always_inline)) {
#pragma unroll
        for (int i = 0; i < UK; ++i)
            if (kkey[i] >= 0) *reinterpret_cast<bf16x8*>(kt + at + kdst[i]) = fk[i];
#pragma unroll
        for (int i = 0; i < UV; ++i)
            if (vkey[i] >= 0) *reinterpret_cast<bf16x8*>(vt + at + vdst[i]) = fv[i];
    };
    // Key tiles start at multiples of 64, and a workgroup begins with one whose number is a multiple of `cycle`, as many as
    // a query tile can see: workgroups that run side by side read the same tiles at about the same time.
    const int t_lo = j_lo / kTileKeys, t_hi = j_hi / kTileKeys, tiles = t_hi - t_lo + 1;
    const int cycle = (p.window + kTileRows - 2) / kTileKeys + 2;
    int tk = (t_lo + cycle - 1) / cycle * cycle;
    tk = tk > t_hi ? t_lo : tk;
    fetch(tk * kTileKeys);
    store(0);
    int now = 0;
    for (int it = 0; it < tiles; ++it, now = buffer - now) {
        const bool more = it + 1 < tiles;
        const int j0 = tk * kTileKeys;
        tk = tk < t_hi ? tk + 1 : t_lo;
        if (more) fetch(tk * kTileKeys);
        __syncthreads();  // this tile is written, and nobody reads the other buffer any more
        // (uniform per wave) does this wave see anything of the tile, and does it see all of it?
        const bool any = j0 <= own_hi && j0 + kTileKeys - 1 > own_lo - p.window;
        const bool all = j0 + kTileKeys - 1 <= own_lo && j0 > own_hi - p.window;
        if (any) {
            f32x4 sc[4][2];
#pragma unroll
            for (int x = 0; x < 4; ++x) {
#pragma unroll
                for (int t = 0; t < 2; ++t) sc[x][t] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
                for (int s = 0; s < NQ; ++s)
                    if (kExact || s < nq) {
                        const bf16x8 a = *reinterpret_cast<const bf16x8*>(kt + now + (16 * x + c) * ks + 32 * s + 8 * g);
#pragma unroll
                        for (int t = 0; t < 2; ++t) sc[x][t] = mfma16(a, q[t][s], sc[x][t]);
                    }
            }
            bf16x8 ph[2][2], pl[2][2];  // [pair of key tiles][query tile]
#pragma unroll
            for (int t = 0; t < 2; ++t) {
                if (!all) {
#pragma unroll
                    for (int x = 0; x < 4; ++x)
#pragma unroll
                        for (int r = 0; r < 4; ++r) {
                            const int j = j0 + 16 * x + 4 * g + r;
                            if (j > own[t] || j <= own[t] - p.window) sc[x][t][r] = kNegInf;
                        }
                }
                // (maximum before the scale, which is positive; scale and difference are one multiply-add)
                float mx = fmaxf(fmaxf(sc[0][t][0], sc[0][t][1]), fmaxf(sc[0][t][2], sc[0][t][3]));
#pragma unroll
                for (int x = 1; x < 4; ++x) mx = fmaxf(mx, fmaxf(fmaxf(sc[x][t][0], sc[x][t][1]), fmaxf(sc[x][t][2], sc[x][t][3])));
                mx = fmaxf(m[t], groups_max(mx) * p.scale_log2);
                const float a = fast_exp2(m[t] - mx);
                m[t] = mx;
                float sum = 0.f;
#pragma unroll
                for (int x = 0; x < 4; ++x) {
                    float w[4];
#pragma unroll
                    for (int r = 0; r < 4; ++r) {
                        w[r] = fast_exp2(__builtin_fmaf(sc[x][t][r], p.scale_log2, -mx));
                        sum += w[r];
                    }
                    const bf16x4 hi = to_bf16x4(w);
#pragma unroll
                    for (int r = 0; r < 4; ++r) w[r] -= (float)hi[r];
                    const bf16x4 lo = to_bf16x4(w);
#pragma unroll
                    for (int r = 0; r < 4; ++r) {
                        ph[x / 2][t][4 * (x % 2) + r] = hi[r];
                        pl[x / 2][t][4 * (x % 2) + r] = lo[r];
                    }
                }
                l[t] = l[t] * a + sum;
                if (__ballot(a != 1.0f) != 0) {
#pragma unroll
                    for (int i = 0; i < NV; ++i)
#pragma unroll
                        for (int r = 0; r < 4; ++r) acc[i][t][r] *= a;
                }
            }
#pragma unroll
            for (int i = 0; i < NV; ++i)
                if (kExact || i < nv) {
#pragma unroll
                    for (int x = 0; x < 2; ++x) {
                        const __bf16* at = vt + now + (32 * x + 4 * g + c / 4) * vs + 16 * i + 4 * (c % 4);
                        const bf16x8 a = join8(lds_read_tr16(reinterpret_cast<const unsigned char*>(at)),
                                               lds_read_tr16(reinterpret_cast<const unsigned char*>(at + 16 * vs)));
#pragma unroll
                        for (int t = 0; t < 2; ++t) {
                            acc[i][t] = mfma16(a, ph[x][t], acc[i][t]);
                            acc[i][t] = mfma16(a, pl[x][t], acc[i][t]);
                        }
                    }
                }
        }
        if (more) store(buffer - now);
    }
#pragma unroll
    for (int t = 0; t < 2; ++t) {
        const float inv = 1.0f / groups_sum(l[t]);
        const int r = wrow + 16 * t + c;
        if (r < row_end) {
#pragma unroll
            for (int i = 0; i < NV; ++i)
                if (kExact || i < nv) {
                    bf16x4 y;
#pragma unroll
                    for (int e = 0; e < 4; ++e) y[e] = (__bf16)(acc[i][t][e] * inv);
                    *reinterpret_cast<bf16x4*>(p.out + (int64_t)r * p.out_rs + (int64_t)h * p.vdim_pad + 16 * i + 4 * g) = y;
                }
        }
    }
}

struct LatentDecode {
    const __bf16 *q_latent, *q_rot, *ring;
    int64_t q_latent_hs, q_rs;
    const int32_t *slot, *pos;
    float* part;  // [rows][heads padded to 16][splits][rank_pad + 4]: sums, the maximum, the sum of weights
    int32_t heads, dim_pad, rot_pad, rank_pad, capacity, nslots, window, rows, splits, tiles_per_split;
    float scale_log2;
};

// grid (splits, groups of 16 heads, rows).  NT: 16-wide tiles of the latent per wave (at most); NU: 16-byte units of a key
// tile per thread, and of steps of 32 of a row (at most; kExact: just so many).
template <int NT, int NU, bool kExact>
__global__ __launch_bounds__(kLatThreads) void latent_decode_kernel(const LatentDecode p) {
    HIP_DYNAMIC_SHARED(unsigned char, dec_lds)
    __shared__ float mx_[kLatWaves][16], sum_[kLatWaves][16];
    const int row = blockIdx.z, tid = threadIdx.x, lane = tid % kWave, wave = tid / kWave, c = lane % 16, g = lane / 16;
    const int lp = kExact ? 32 * NU : p.rank_pad + p.rot_pad, steps = lp / 32, nt = kExact ? kLatWaves * NT : p.rank_pad / 16, ks = lp + 8, ps = kTileKeys + 8;
    __bf16* const kt = reinterpret_cast<__bf16*>(dec_lds);  // [64 keys][ks]
    __bf16* const qt = kt + kTileKeys * ks;                 // [16 heads][ks]
    __bf16* const pt = qt + 16 * ks;                        // [2 terms][16 heads][ps]
    const int pos = p.pos[row];
    int slot = p.slot[row];
    if (slot >= p.nslots) slot = -1;
    const bool live = slot >= 0 && pos >= 0;
    const int units = kTileKeys * lp / 8, upk = lp / 8;
    const __bf16* const ring = p.ring + (int64_t)(slot < 0 ? 0 : slot) * p.capacity * lp;
    int lo = pos - p.window + 1;
    lo = lo < 0 ? 0 : lo;
    const int begin = lo + blockIdx.x * p.tiles_per_split * kTileKeys;
    int end = begin + p.tiles_per_split * kTileKeys - 1;
    end = end < pos ? end : pos;
    if (!live) end = begin - 1;
    bf16x8 fk[NU];
    int key[NU], dst[NU];
#pragma unroll
    for (int i = 0; i < NU; ++i) {
        const int u = tid + kLatThreads * i;
        key[i] = kExact || u < units ? u / upk : -1;
        dst[i] = (u / upk) * ks + 8 * (u % upk);
    }
    // a key's row of the ring: the first one's, advanced, wrapped at most once per tile (a tile is not longer than the ring,
    // or the positions past `end` repeat the last)
    auto fetch = [&](int j0) __attribute__((always_inline)) {
        const int r0 = j0 % p.capacity;
#pragma unroll
        for (int i = 0; i < NU; ++i) {
            if (key[i] >= 0) {
                int r = r0 + (j0 + key[i] < end ? key[i] : end - j0);
                r = r >= p.capacity ? r - p.capacity : r;
                fk[i] = *reinterpret_cast<const bf16x8*>(ring + (int64_t)r * lp + dst[i] - key[i] * ks);
            }
        }
    };
    if (begin <= end) fetch(begin);
    for (int u = tid; u < 16 * upk; u += kLatThreads) {
        int h = blockIdx.y * 16 + u / upk;
        h = h < p.heads ? h : p.heads - 1;  // heads past the last one repeat it; nobody reads them
        const int x = 8 * (u % upk);
        const __bf16* src = x < p.rank_pad ? p.q_latent + h * p.q_latent_hs + (int64_t)row * p.rank_pad + x
                                           : p.q_rot + (int64_t)row * p.q_rs + (int64_t)h * (p.dim_pad + p.rot_pad) + x - p.rank_pad;
        *reinterpret_cast<bf16x8*>(qt + (u / upk) * ks + x) = *reinterpret_cast<const bf16x8*>(src);
    }
    f32x4 acc[NT];
#pragma unroll
    for (int i = 0; i < NT; ++i) acc[i] = f32x4{0.f, 0.f, 0.f, 0.f};
    float m = kNoScore, l = 0.f;
    for (int j0 = begin; j0 <= end; j0 += kTileKeys) {
#pragma unroll
        for (int i = 0; i < NU; ++i)
            if (key[i] >= 0) *reinterpret_cast<bf16x8*>(kt + dst[i]) = fk[i];
        __syncthreads();
        if (j0 + kTileKeys <= end) fetch(j0 + kTileKeys);
        // scores of this wave's sixteen keys: register r of lane (c, g) is key 16 wave + 4 g + r, head c
        f32x4 sc = f32x4{0.f, 0.f, 0.f, 0.f}, sc2 = sc;
#pragma unroll
        for (int s = 0; s < NU; ++s)  // (a row has as many steps of 32 as a thread has units of a tile)
            if (kExact || s < steps) {
                const bf16x8 a = *reinterpret_cast<const bf16x8*>(kt + (16 * wave + c) * ks + 32 * s + 8 * g);
                const bf16x8 b = *reinterpret_cast<const bf16x8*>(qt + c * ks + 32 * s + 8 * g);
                if (s % 2) sc2 = mfma16(a, b, sc2);
                else sc = mfma16(a, b, sc);
            }
#pragma unroll
        for (int r = 0; r < 4; ++r) sc[r] += sc2[r];
        float mw = kNoScore;
#pragma unroll
        for (int r = 0; r < 4; ++r) {
            sc[r] = j0 + 16 * wave + 4 * g + r <= end ? sc[r] * p.scale_log2 : kNegInf;
            mw = fmaxf(mw, sc[r]);
        }
        mw = groups_max(mw);
        if (g == 0) mx_[wave][c] = mw;
        __syncthreads();
        const float mn = fmaxf(m, fmaxf(fmaxf(mx_[0][c], mx_[1][c]), fmaxf(mx_[2][c], mx_[3][c])));
        const float a = fast_exp2(m - mn);
        m = mn;
        bf16x4 hi, rest;
        l *= a;
#pragma unroll
        for (int r = 0; r < 4; ++r) {
            const float w = fast_exp2(sc[r] - mn);
            l += w;
            hi[r] = (__bf16)w;
            rest[r] = (__bf16)(w - (float)hi[r]);
        }
        *reinterpret_cast<bf16x4*>(pt + c * ps + 16 * wave + 4 * g) = hi;
        *reinterpret_cast<bf16x4*>(pt + (16 + c) * ps + 16 * wave + 4 * g) = rest;
#pragma unroll
        for (int i = 0; i < NT; ++i)
#pragma unroll
            for (int r = 0; r < 4; ++r) acc[i][r] *= a;
        __syncthreads();
#pragma unroll
        for (int x = 0; x < 2; ++x) {
            const __bf16* pr = pt + c * ps + 32 * x + 4 * g;
            const bf16x8 ph = join8(*reinterpret_cast<const bf16x4*>(pr), *reinterpret_cast<const bf16x4*>(pr + 16));
            const bf16x8 pl = join8(*reinterpret_cast<const bf16x4*>(pr + 16 * ps), *reinterpret_cast<const bf16x4*>(pr + 16 * ps + 16));
#pragma unroll
            for (int i = 0; i < NT; ++i) {
                const int t = wave + kLatWaves * i;
                if (kExact || t < nt) {
                    const __bf16* at = kt + (32 * x + 4 * g + c / 4) * ks + 16 * t + 4 * (c % 4);
                    const bf16x8 v = join8(lds_read_tr16(reinterpret_cast<const unsigned char*>(at)),
                                           lds_read_tr16(reinterpret_cast<const unsigned char*>(at + 16 * ks)));
                    acc[i] = mfma16(v, ph, acc[i]);
                    acc[i] = mfma16(v, pl, acc[i]);
                }
            }
        }
        __syncthreads();
    }
    l = groups_sum(l);
    if (g == 0) sum_[wave][c] = l;
    __syncthreads();
    const int hp = gridDim.y * 16;
    float* const out = p.part + (((int64_t)row * hp + blockIdx.y * 16 + c) * p.splits + blockIdx.x) * (p.rank_pad + 4);
    if (begin <= end) {
#pragma unroll
        for (int i = 0; i < NT; ++i) {
            const int t = wave + kLatWaves * i;
            if (t < nt) *reinterpret_cast<f32x4*>(out + 16 * t + 4 * g) = acc[i];
        }
    }
    if (tid < 16) {
        out[p.rank_pad] = m;
        out[p.rank_pad + 1] = (sum_[0][c] + sum_[1][c]) + (sum_[2][c] + sum_[3][c]);  // 0: nothing seen, no sums written
    }
}

// grid (heads, rows); four latent columns per thread
__global__ __launch_bounds__(kLatThreads) void latent_merge_kernel(const float* part, int hp, int splits, int rank_pad, int rows, __bf16* out_packed,
                                                                   __bf16* out_rows) {
    const int h = blockIdx.x, row = blockIdx.y, i = 4 * threadIdx.x, ps = rank_pad + 4;
    const float* const base = part + ((int64_t)row * hp + h) * splits * ps;
    if (i >= rank_pad) return;
    float m = kNoScore, l = 0.f;
    f32x4 y = {0.f, 0.f, 0.f, 0.f};
    for (int s0 = 0; s0 < splits; s0 += 4) {
        f32x4 v[4];
        float vm[4], vl[4];
#pragma unroll
        for (int x = 0; x < 4; ++x) {
            const float* p = base + (int64_t)(s0 + x < splits ? s0 + x : splits - 1) * ps;
            v[x] = *reinterpret_cast<const f32x4*>(p + i);
            vm[x] = p[rank_pad];
            vl[x] = s0 + x < splits ? p[rank_pad + 1] : 0.f;
        }
#pragma unroll
        for (int x = 0; x < 4; ++x) {
            if (!(vl[x] > 0.f)) continue;  // saw nothing: its sums were not written
            const float mn = fmaxf(m, vm[x]), a = fast_exp2(m - mn), b = fast_exp2(vm[x] - mn);
            m = mn;
            l = l * a + vl[x] * b;
#pragma unroll
            for (int e = 0; e < 4; ++e) y[e] = y[e] * a + v[x][e] * b;
        }
    }
    const float inv = l > 0.f ? 1.0f / l : 0.f;
    bf16x4 o;
#pragma unroll
    for (int e = 0; e < 4; ++e) o[e] = (__bf16)(y[e] * inv);
    if (out_packed) *reinterpret_cast<bf16x4*>(out_packed + (int64_t)h * 32 * rank_pad + rows_form_elem(row, i)) = o;
    if (out_rows) *reinterpret_cast<bf16x4*>(out_rows + ((int64_t)h * rows + row) * rank_pad + i) = o;
}

int check_layer(const tah_latent_layer* L) {
    if (!L) return TAH_E_NULL;
    if (L->heads <= 0 || L->heads > 65535 || L->dim_pad <= 0 || L->dim_pad % 32 != 0 || L->rot_dim < 0 || L->rot_dim % 2 != 0 ||
        L->rot_pad < L->rot_dim || L->rot_pad % 32 != 0 || L->rank <= 0 || L->rank_pad < L->rank || L->rank_pad % 32 != 0 || L->vdim_pad <= 0 ||
        L->vdim_pad % 16 != 0 || L->capacity <= 0 || L->nslots <= 0 || L->window <= 0 || (L->dtype != TAH_DT_BF16 && L->dtype != TAH_DT_F32))
        return TAH_E_SHAPE;
    if (L->rank_pad > kLatThreads * kAttValues || L->vdim_pad > kLatThreads * kAttValues || L->dim_pad + L->rot_pad > 8192 || L->rot_pad > 4096) return TAH_E_SHAPE;
    if (!L->ring) return TAH_E_NULL;
    if (!aligned_16(L->ring)) return TAH_E_ALIGN;
    return TAH_OK;
}
int check_portions(const tah_portions* p) {
    if (!p) return TAH_E_NULL;
    if (p->nseq < 0 || p->rows < 0) return TAH_E_SHAPE;
    if (p->nseq > 0 && p->rows > 0 && (!p->cu || !p->slot || !p->pos0 || !p->row_seq)) return TAH_E_NULL;
    return TAH_OK;
}
void launch_attend_rows(const AttendRows& p, int heads, int dtype, hipStream_t st) {
    const size_t lds = (size_t)(p.n1 + p.n2) * sizeof(float);
    if (dtype == TAH_DT_BF16) hipLaunchKernelGGL((attend_rows_kernel<__bf16>), dim3(p.rows, heads), dim3(kLatThreads), lds, st, p);
    else hipLaunchKernelGGL((attend_rows_kernel<float>), dim3(p.rows, heads), dim3(kLatThreads), lds, st, p);
}
size_t elem_bytes(int dtype) { return dtype == TAH_DT_BF16 ? 2 : 4; }

template <int NQ, int NV, int W, bool kExact>
int launch_attend_tile(AttendTile p, int rows, hipStream_t st) {
    const size_t lds = (size_t)2 * kTileKeys * (p.dim_pad + p.rot_pad + 8 + p.vdim_pad + 16) * 2;
    if (lds > 65536 && hipFuncSetAttribute(reinterpret_cast<const void*>(&attend_tile_kernel<NQ, NV, W, kExact>),
                                           hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds) != hipSuccess)
        return TAH_E_LAUNCH;
    p.slots = rows / (32 * W) + p.nseq;
    hipLaunchKernelGGL((attend_tile_kernel<NQ, NV, W, kExact>), dim3((unsigned)(p.slots * p.heads)), dim3(W * kWave), lds, st, p);
    return launch_status();
}

// how a decode call splits its window: enough workgroups for the chip, whole tiles of 64 keys each
constexpr int kDecodeGroups = 256;
void decode_split(int heads, int rows, int window, int& splits, int& tiles_per_split) {
    const int tiles = (window + kTileKeys - 1) / kTileKeys, groups = rows * ((heads + 15) / 16);
    int want = groups > 0 ? kDecodeGroups / groups : 1;
    want = want < 1 ? 1 : (want > tiles ? tiles : want);
    tiles_per_split = (tiles + want - 1) / want;
    splits = (tiles + tiles_per_split - 1) / tiles_per_split;
}
size_t decode_lds(int lp) { return ((size_t)(kTileKeys + 16) * (lp + 8) + 2 * 16 * (kTileKeys + 8)) * 2; }
constexpr size_t kLdsBytes = 160 * 1024 - 1024;  // a compute unit's LDS, less the kernel's static part
bool decode_on_tiles(const tah_latent_layer* L) { return L->dtype == TAH_DT_BF16 && decode_lds(L->rank_pad + L->rot_pad) <= kLdsBytes; }

template <int NT, int NU, bool kExact>
int launch_latent_decode(const LatentDecode& p, hipStream_t st) {
    const size_t lds = decode_lds(p.rank_pad + p.rot_pad);
    if (lds > 65536 && hipFuncSetAttribute(reinterpret_cast<const void*>(&latent_decode_kernel<NT, NU, kExact>), hipFuncAttributeMaxDynamicSharedMemorySize,
                                           (int)lds) != hipSuccess)
        return TAH_E_LAUNCH;
    hipLaunchKernelGGL((latent_decode_kernel<NT, NU, kExact>), dim3(p.splits, (p.heads + 15) / 16, p.rows), dim3(kLatThreads), lds, st, p);
    return launch_status();
}

}  // namespace
}  // namespace tah

extern "C" int tah_latent_prep(const tah_latent_layer* L, const tah_latent_prep_args* a, tah_stream_t stream) {
    using namespace tah;
    if (const int rc = check_layer(L)) return rc;
    if (!a) return TAH_E_NULL;
    if (a->rows < 0 || a->q_col < 0 || a->q_col % 8 != 0 || a->table_rows <= 0 || a->proj_row_stride % 8 != 0) return TAH_E_SHAPE;
    if (a->q_packed && (a->rows > 32 || L->dtype != TAH_DT_BF16)) return TAH_E_SHAPE;
    if (a->rows == 0) return TAH_OK;
    if (!a->proj || !a->pos || (L->rot_dim > 0 && (!a->cos || !a->sin)) || (a->dkv_col >= 0 && !a->norm)) return TAH_E_NULL;
    if (!aligned_16(a->proj) || !aligned_16(a->rows_out) || !aligned_16(a->q_packed) || !aligned_16(a->q_rows)) return TAH_E_ALIGN;
    hipStream_t st = static_cast<hipStream_t>(stream);
    if (L->dtype == TAH_DT_BF16) hipLaunchKernelGGL((latent_prep_kernel<__bf16>), dim3(a->rows), dim3(kLatThreads), 0, st, *L, *a);
    else hipLaunchKernelGGL((latent_prep_kernel<float>), dim3(a->rows), dim3(kLatThreads), 0, st, *L, *a);
    return launch_status();
}

extern "C" int tah_latent_context(const tah_latent_layer* L, const tah_portions* p, const int32_t* cu_k, int32_t ctx_rows, const void* new_rows,
                                  void* ctx, tah_stream_t stream) {
    using namespace tah;
    if (const int rc = check_layer(L)) return rc;
    if (const int rc = check_portions(p)) return rc;
    if (ctx_rows < 0) return TAH_E_SHAPE;
    if (p->rows == 0 || p->nseq == 0) return TAH_OK;
    if (!cu_k || !new_rows || (ctx_rows > 0 && !ctx)) return TAH_E_NULL;
    if (!aligned_16(new_rows) || !aligned_16(ctx)) return TAH_E_ALIGN;
    hipStream_t st = static_cast<hipStream_t>(stream);
    const dim3 gc((ctx_rows + kLatWaves - 1) / kLatWaves), ga((p->rows + kLatWaves - 1) / kLatWaves);
    if (L->dtype == TAH_DT_BF16) {
        if (ctx_rows > 0)
            hipLaunchKernelGGL((latent_context_kernel<__bf16>), gc, dim3(kLatThreads), 0, st, *L, *p, cu_k, (int)ctx_rows,
                               static_cast<const __bf16*>(new_rows), static_cast<__bf16*>(ctx));
        hipLaunchKernelGGL((latent_append_kernel<__bf16>), ga, dim3(kLatThreads), 0, st, *L, *p, static_cast<const __bf16*>(new_rows));
    } else {
        if (ctx_rows > 0)
            hipLaunchKernelGGL((latent_context_kernel<float>), gc, dim3(kLatThreads), 0, st, *L, *p, cu_k, (int)ctx_rows,
                               static_cast<const float*>(new_rows), static_cast<float*>(ctx));
        hipLaunchKernelGGL((latent_append_kernel<float>), ga, dim3(kLatThreads), 0, st, *L, *p, static_cast<const float*>(new_rows));
    }
    return launch_status();
}

extern "C" int tah_latent_attend(const tah_latent_layer* L, const tah_portions* p, const int32_t* cu_k, int32_t max_rows, const void* q,
                                 int64_t q_rs, const void* k, int64_t k_rs, const void* v, int64_t v_rs, const void* ctx, void* out,
                                 int64_t out_rs, tah_stream_t stream) {
    using namespace tah;
    if (const int rc = check_layer(L)) return rc;
    if (const int rc = check_portions(p)) return rc;
    if (max_rows < 0 || q_rs % 8 != 0 || k_rs % 8 != 0 || v_rs % 8 != 0 || out_rs % 8 != 0) return TAH_E_SHAPE;
    if (p->rows == 0 || p->nseq == 0) return TAH_OK;
    if (!cu_k || !q || !k || !v || !ctx || !out) return TAH_E_NULL;
    if (!aligned_16(q) || !aligned_16(k) || !aligned_16(v) || !aligned_16(ctx) || !aligned_16(out)) return TAH_E_ALIGN;
    const int nq = (L->dim_pad + L->rot_pad) / 32, nv = (L->vdim_pad + 15) / 16;
    if (L->dtype == TAH_DT_BF16 && nq <= 10 && nv <= 16 && L->scale > 0.f) {
        AttendTile t{};
        t.q = static_cast<const __bf16*>(q); t.k = static_cast<const __bf16*>(k); t.v = static_cast<const __bf16*>(v);
        t.ctx = static_cast<const __bf16*>(ctx) + L->rank_pad;
        t.q_rs = q_rs; t.k_rs = k_rs; t.v_rs = v_rs; t.ctx_rs = L->rank_pad + L->rot_pad;
        t.out = static_cast<__bf16*>(out); t.out_rs = out_rs;
        t.cu = p->cu; t.cu_k = cu_k; t.nseq = p->nseq;
        t.dim_pad = L->dim_pad; t.rot_pad = L->rot_pad; t.vdim_pad = L->vdim_pad; t.window = L->window;
        t.scale_log2 = L->scale * kLog2e;
        hipStream_t st = static_cast<hipStream_t>(stream);
        t.heads = L->heads;
        if (nq == 6 && nv == 8) return launch_attend_tile<6, 8, 8, true>(t, p->rows, st);
        if (nq <= 4 && nv <= 4) return launch_attend_tile<4, 4, 8, false>(t, p->rows, st);
        if (nq <= 6 && nv <= 8) return launch_attend_tile<6, 8, 8, false>(t, p->rows, st);
        return launch_attend_tile<10, 16, 4, false>(t, p->rows, st);
    }
    AttendRows a{};
    a.q1 = q; a.q1_rs = q_rs; a.q1_hs = L->dim_pad + L->rot_pad; a.n1 = L->dim_pad;
    a.q2 = static_cast<const char*>(q) + (size_t)L->dim_pad * elem_bytes(L->dtype); a.q2_rs = q_rs; a.q2_hs = a.q1_hs; a.n2 = L->rot_pad;
    a.k1 = k; a.k1_rs = k_rs; a.k1_hs = L->dim_pad;
    a.k2 = static_cast<const char*>(ctx) + (size_t)L->rank_pad * elem_bytes(L->dtype); a.k2_rs = L->rank_pad + L->rot_pad;
    a.v = v; a.v_rs = v_rs; a.v_hs = L->vdim_pad; a.nv = L->vdim_pad;
    a.cu = p->cu; a.cu_k = cu_k; a.pos0 = p->pos0; a.row_seq = p->row_seq;
    a.window = L->window; a.rows = p->rows; a.scale = L->scale;
    a.out = out; a.out_rs = out_rs; a.out_hs = L->vdim_pad;
    launch_attend_rows(a, L->heads, L->dtype, static_cast<hipStream_t>(stream));
    return launch_status();
}

extern "C" size_t tah_latent_decode_workspace(const tah_latent_layer* L, int32_t rows) {
    if (tah::check_layer(L) != TAH_OK || rows <= 0 || !tah::decode_on_tiles(L)) return 0;
    const size_t groups = (size_t)rows * ((L->heads + 15) / 16);  // (rank_pad <= 4 * kLatThreads: one pass of the merge)
    return (groups > tah::kDecodeGroups ? groups : (size_t)tah::kDecodeGroups) * 16 * (L->rank_pad + 4) * sizeof(float);  // enough for fewer rows too
}

extern "C" int tah_latent_decode(const tah_latent_layer* L, const int32_t* slot, const int32_t* pos, int32_t rows, const void* q_latent,
                                 int64_t q_latent_hs, const void* q, int64_t q_rs, void* out_packed, void* out_rows, void* workspace,
                                 size_t workspace_bytes, tah_stream_t stream) {
    using namespace tah;
    if (const int rc = check_layer(L)) return rc;
    if (rows < 0 || (out_packed && rows > 32) || q_rs % 8 != 0 || q_latent_hs % 8 != 0 || L->window > L->capacity) return TAH_E_SHAPE;
    if (rows == 0) return TAH_OK;
    if (!slot || !pos || !q_latent || !q || (!out_packed && !out_rows)) return TAH_E_NULL;
    if (!aligned_16(q_latent) || !aligned_16(q) || !aligned_16(out_packed) || !aligned_16(out_rows)) return TAH_E_ALIGN;
    if (decode_on_tiles(L)) {
        LatentDecode d{};
        d.q_latent = static_cast<const __bf16*>(q_latent); d.q_latent_hs = q_latent_hs;
        d.q_rot = static_cast<const __bf16*>(q) + L->dim_pad; d.q_rs = q_rs;
        d.ring = static_cast<const __bf16*>(L->ring); d.slot = slot; d.pos = pos; d.part = static_cast<float*>(workspace);
        d.heads = L->heads; d.dim_pad = L->dim_pad; d.rot_pad = L->rot_pad; d.rank_pad = L->rank_pad; d.capacity = L->capacity; d.nslots = L->nslots;
        d.window = L->window; d.rows = rows; d.scale_log2 = L->scale * kLog2e;
        decode_split(L->heads, rows, L->window, d.splits, d.tiles_per_split);
        const int hp = (L->heads + 15) / 16 * 16;
        if (!workspace || workspace_bytes < (size_t)rows * hp * d.splits * (L->rank_pad + 4) * sizeof(float)) return TAH_E_WORKSPACE;
        hipStream_t st = static_cast<hipStream_t>(stream);
        const int lp = L->rank_pad + L->rot_pad;
        int rc;
        if (lp == 576 && L->rank_pad == 512) rc = launch_latent_decode<8, 18, true>(d, st);
        else if (lp <= 128) rc = launch_latent_decode<2, 4, false>(d, st);
        else if (lp <= 320) rc = launch_latent_decode<5, 10, false>(d, st);
        else if (lp <= 576) rc = launch_latent_decode<9, 18, false>(d, st);
        else rc = launch_latent_decode<16, 32, false>(d, st);
        if (rc != TAH_OK) return rc;
        hipLaunchKernelGGL(latent_merge_kernel, dim3(L->heads, rows), dim3(kLatThreads), 0, st, static_cast<const float*>(workspace), hp, (int)d.splits,
                           (int)L->rank_pad, (int)rows, static_cast<__bf16*>(out_packed), static_cast<__bf16*>(out_rows));
        return launch_status();
    }
    AttendRows a{};
    a.q1 = q_latent; a.q1_rs = L->rank_pad; a.q1_hs = q_latent_hs; a.n1 = L->rank_pad;
    a.q2 = static_cast<const char*>(q) + (size_t)L->dim_pad * elem_bytes(L->dtype); a.q2_rs = q_rs; a.q2_hs = L->dim_pad + L->rot_pad; a.n2 = L->rot_pad;
    a.k1 = L->ring; a.k1_rs = L->rank_pad + L->rot_pad; a.k1_hs = 0;
    a.k2 = static_cast<const char*>(L->ring) + (size_t)L->rank_pad * elem_bytes(L->dtype); a.k2_rs = a.k1_rs;
    a.v = L->ring; a.v_rs = a.k1_rs; a.v_hs = 0; a.nv = L->rank_pad;
    a.slot = slot; a.pos = pos; a.capacity = L->capacity; a.nslots = L->nslots;
    a.window = L->window; a.rows = rows; a.scale = L->scale;
    a.out = out_rows; a.out_rs = L->rank_pad; a.out_hs = (int64_t)rows * L->rank_pad;
    a.out_packed = out_packed;
    launch_attend_rows(a, L->heads, L->dtype, static_cast<hipStream_t>(stream));
    return launch_status();
}
