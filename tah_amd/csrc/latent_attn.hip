// Sliding-window latent attention, gfx950.  A token's keys and values of all heads are linear in one latent c [rank];
// what is cached is c and a rotated key part shared by the heads, one row per token, in a ring per sequence that is
// as long as the widest window that reads it.
//
//  * latent_prep_kernel: projections of a step's or a portion's rows -> normed latents and rotated key part (into the
//    ring, or packed for tah_latent_context), rotated query part, and the unrotated query part in the operand order of
//    the per-head products.
//  * latent_context_kernel / latent_append_kernel: the rows a batch of portions can see, packed (old ones from the
//    ring, new ones from the portion), then the new rows into the ring.
//  * attend_rows_kernel: one workgroup per (query, head), any sizes, either element type.
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
    (void)L; (void)rows;
    return 0;
}

extern "C" int tah_latent_decode(const tah_latent_layer* L, const int32_t* slot, const int32_t* pos, int32_t rows, const void* q_latent,
                                 int64_t q_latent_hs, const void* q, int64_t q_rs, void* out_packed, void* out_rows, void* workspace,
                                 size_t workspace_bytes, tah_stream_t stream) {
    using namespace tah;
    (void)workspace; (void)workspace_bytes;
    if (const int rc = check_layer(L)) return rc;
    if (rows < 0 || (out_packed && rows > 32) || q_rs % 8 != 0 || q_latent_hs % 8 != 0 || L->window > L->capacity) return TAH_E_SHAPE;
    if (rows == 0) return TAH_OK;
    if (!slot || !pos || !q_latent || !q || (!out_packed && !out_rows)) return TAH_E_NULL;
    if (!aligned_16(q_latent) || !aligned_16(q) || !aligned_16(out_packed) || !aligned_16(out_rows)) return TAH_E_ALIGN;
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
