// Bindings of include/tah_mixers.h: each checks its tensors, fills the C structs and calls the entry point on torch's
// current HIP stream.
#include "torch_ext.h"

namespace py = pybind11;

namespace tah_ext {
namespace {

at::ScalarType elem_type(int32_t dtype) { return dtype == TAH_DT_BF16 ? at::kBFloat16 : at::kFloat; }
int32_t dtype_of(const Tensor& t, const char* what) {
    TORCH_CHECK(t.scalar_type() == at::kBFloat16 || t.scalar_type() == at::kFloat, what, " must be bf16 or float32");
    return t.scalar_type() == at::kBFloat16 ? TAH_DT_BF16 : TAH_DT_F32;
}
// contiguous tensor of a type and (n >= 0) a number of elements
void flat(const Tensor& t, at::ScalarType ty, int64_t n, const char* what) {
    TORCH_CHECK(t.scalar_type() == ty && t.is_contiguous() && (n < 0 || t.numel() == n), what, ": a contiguous tensor of ", n, " elements of ", ty,
                " expected, got ", t.numel(), " of ", t.scalar_type());
}
void flat(const optional<Tensor>& t, at::ScalarType ty, int64_t n, const char* what) { if (t.has_value()) flat(*t, ty, n, what); }
// matrix [rows, >= cols] with contiguous rows
int64_t matrix(const Tensor& t, at::ScalarType ty, int64_t rows, int64_t cols, const char* what) {
    TORCH_CHECK(t.dim() == 2 && t.scalar_type() == ty && t.size(0) >= rows && t.size(1) >= cols && (t.numel() == 0 || t.stride(1) == 1), what, ": a [", rows,
                ", ", cols, "] matrix of ", ty, " with contiguous rows expected");
    return t.size(0) > 1 ? t.stride(0) : t.size(1);
}
template <class T> T* at_(const Tensor& t) { return static_cast<T*>(mptr(t)); }
template <class T> T* at_(const optional<Tensor>& t) { return t.has_value() ? static_cast<T*>(mptr(*t)) : nullptr; }
void* any(const optional<Tensor>& t) { return t.has_value() ? mptr(*t) : nullptr; }

// A batch of portions: what tah_portions points at.
struct Portions {
    Tensor cu, slot, pos0, row_seq;
    Portions(Tensor cu_, Tensor slot_, Tensor pos0_, Tensor row_seq_) : cu(cu_), slot(slot_), pos0(pos0_), row_seq(row_seq_) {
        flat(cu, at::kInt, slot.numel() + 1, "Portions: cu"); flat(slot, at::kInt, -1, "Portions: slot");
        flat(pos0, at::kInt, slot.numel(), "Portions: pos0"); flat(row_seq, at::kInt, -1, "Portions: row_seq");
    }
    tah_portions c(Dev& d) const {
        d.see(cu); d.see(slot); d.see(pos0); d.see(row_seq);
        return {at_<int32_t>(cu), at_<int32_t>(slot), at_<int32_t>(pos0), at_<int32_t>(row_seq), (int32_t)slot.numel(), (int32_t)row_seq.numel()};
    }
};

void embed_rows(const Tensor& tok, const Tensor& embed, const Tensor& x, const optional<Tensor>& xe, const optional<Tensor>& x_packed,
                const optional<Tensor>& pos, const optional<Tensor>& finished, const optional<Tensor>& slot, const optional<Tensor>& q_pos,
                const optional<Tensor>& active, int64_t slot_base, double scale) {
    need_lib();
    Dev d; d.see(tok); d.see(embed); d.see(x); d.see(xe); d.see(x_packed); d.see(pos); d.see(finished); d.see(slot); d.see(q_pos); d.see(active);
    const int64_t rows = tok.numel(), cols = embed.size(1);
    tah_embed_rows_args a{};
    a.dtype = dtype_of(embed, "embed_rows: embed");
    flat(tok, at::kLong, rows, "embed_rows: tok");
    flat(embed, embed.scalar_type(), -1, "embed_rows: embed");
    flat(x, at::kFloat, rows * cols, "embed_rows: x");
    flat(xe, embed.scalar_type(), rows * cols, "embed_rows: xe");
    flat(x_packed, at::kBFloat16, 32 * cols, "embed_rows: x_packed");
    flat(pos, at::kInt, rows, "embed_rows: pos"); flat(finished, at::kBool, rows, "embed_rows: finished");
    flat(slot, at::kInt, rows, "embed_rows: slot"); flat(q_pos, at::kInt, rows, "embed_rows: q_pos"); flat(active, at::kBool, rows, "embed_rows: active");
    a.tok = at_<int64_t>(tok); a.pos = at_<int32_t>(pos); a.finished = at_<uint8_t>(finished); a.embed = ptr(embed); a.x = at_<float>(x);
    a.xe = any(xe); a.x_packed = any(x_packed); a.slot = at_<int32_t>(slot); a.q_pos = at_<int32_t>(q_pos); a.active = at_<uint8_t>(active);
    a.rows = (int32_t)rows; a.vocab = (int32_t)embed.size(0); a.cols = (int32_t)cols; a.slot_base = (int32_t)slot_base;
    a.scale = (float)scale;
    check_rc(g.embed_rows(&a, d.stream()), "tah_embed_rows");
}

// A short causal convolution of a sublayer's input: its taps [taps, cols] and the slots' last inputs [slots, taps, cols].
struct InputConv {
    Tensor w, state;
    InputConv(Tensor w_, Tensor state_) : w(w_), state(state_) {
        TORCH_CHECK(w.dim() == 2 && state.dim() == 3 && state.size(1) == w.size(0) && state.size(2) == w.size(1),
                    "InputConv: w [taps, cols], state [slots, taps, cols]");
        flat(w, at::kFloat, -1, "InputConv: w");
        dtype_of(state, "InputConv: state");
        TORCH_CHECK(state.is_contiguous(), "InputConv: state must be contiguous");
    }
};

void residual_norm(const Tensor& x, const optional<Tensor>& coef, int64_t width, double eps, const optional<Tensor>& y, const optional<Tensor>& y_scale,
                   const optional<Tensor>& experts, const optional<Tensor>& index, const optional<Tensor>& weight, const optional<Tensor>& xe,
                   const optional<Tensor>& x_packed, const optional<Tensor>& next_coef, const optional<Tensor>& normed,
                   const optional<Tensor>& normed_packed, int64_t index_scale, int64_t index_row, int64_t groups, int64_t group_cols,
                   const InputConv* conv, const optional<Tensor>& slot, const optional<Tensor>& pos) {
    need_lib();
    Dev d; d.see(x); d.see(coef); d.see(y); d.see(y_scale); d.see(experts); d.see(index); d.see(weight); d.see(xe); d.see(x_packed);
    d.see(next_coef); d.see(normed); d.see(normed_packed); d.see(slot); d.see(pos);
    TORCH_CHECK(x.dim() == 2, "residual_norm: x must be [rows, cols]");
    const int64_t rows = x.size(0), cols = x.size(1);
    // (the element type is that of whatever is given in it)
    const optional<Tensor>* const elems[] = {&y, &experts, &xe, &normed, &x_packed, &normed_packed};
    const Tensor* elem = nullptr;
    for (const auto* t : elems)
        if (!elem && t->has_value()) elem = &**t;
    TORCH_CHECK(elem, "residual_norm: nothing to add and nothing to write");
    const at::ScalarType ty = elem->scalar_type();
    tah_residual_norm_args a{};
    a.dtype = dtype_of(*elem, "residual_norm: y");
    flat(x, at::kFloat, rows * cols, "residual_norm: x");
    flat(coef, at::kFloat, cols, "residual_norm: coef"); flat(next_coef, at::kFloat, cols, "residual_norm: next_coef");
    flat(xe, ty, rows * cols, "residual_norm: xe"); flat(normed, ty, rows * cols, "residual_norm: normed");
    flat(x_packed, at::kBFloat16, 32 * cols, "residual_norm: x_packed"); flat(normed_packed, at::kBFloat16, 32 * cols, "residual_norm: normed_packed");
    flat(y_scale, at::kFloat, rows, "residual_norm: y_scale");
    if (y.has_value()) { a.y = ptr(*y); a.y_row_stride = matrix(*y, ty, rows, cols, "residual_norm: y"); }
    if (experts.has_value()) {
        TORCH_CHECK(index.has_value() && weight.has_value() && index->dim() == 2, "residual_norm: experts need index and weight [rows, top]");
        a.top = (int32_t)index->size(1);
        flat(*index, at::kInt, rows * a.top, "residual_norm: index"); flat(*weight, at::kFloat, rows * a.top, "residual_norm: weight");
        a.experts = ptr(*experts); a.experts_row_stride = matrix(*experts, ty, 1, cols, "residual_norm: experts");
        a.index_scale = (int32_t)index_scale; a.index_row = (int32_t)index_row;
        a.index = at_<int32_t>(*index); a.weight = at_<float>(*weight);
    }
    a.y_scale = at_<float>(y_scale); a.coef = at_<float>(coef); a.next_coef = at_<float>(next_coef); a.x = at_<float>(x);
    a.xe = any(xe); a.x_packed = any(x_packed); a.normed = any(normed); a.normed_packed = any(normed_packed);
    a.rows = (int32_t)rows; a.width = (int32_t)width; a.cols = (int32_t)cols; a.eps = (float)eps;
    a.groups = (int32_t)groups; a.group_cols = (int32_t)group_cols;
    if (conv) {
        d.see(conv->w); d.see(conv->state);
        TORCH_CHECK(slot.has_value() && pos.has_value() && conv->w.size(1) == cols && conv->state.scalar_type() == ty,
                    "residual_norm: the convolution needs slot, pos and rows of its own width and type");
        flat(slot, at::kInt, rows, "residual_norm: slot"); flat(pos, at::kInt, rows, "residual_norm: pos");
        a.conv = at_<float>(conv->w); a.conv_state = mptr(conv->state); a.slot = at_<int32_t>(slot); a.pos = at_<int32_t>(pos);
        a.taps = (int32_t)conv->w.size(0); a.nslots = (int32_t)conv->state.size(0);
    }
    check_rc(g.residual_norm(&a, d.stream()), "tah_residual_norm");
}

Tensor activate_rows(const Tensor& in, int64_t kind, const optional<Tensor>& out_, double c0, double c1) {
    need_lib();
    Dev d; d.see(in); d.see(out_);
    TORCH_CHECK(in.dim() == 2 && (in.numel() == 0 || in.stride(1) == 1), "activate_rows: a matrix with contiguous rows expected");
    const int64_t rows = in.size(0), cols = kind == TAH_ROWS_SILU_MUL || kind == TAH_ROWS_CLAMPED_GATE ? in.size(1) / 2 : in.size(1);
    Tensor out = out_.has_value() ? *out_ : at::empty({rows, cols}, in.options());
    const int64_t rs = matrix(out, in.scalar_type(), rows, cols, "activate_rows: out");
    check_rc(g.activate_rows(ptr(in), rows > 1 ? in.stride(0) : in.size(1), mptr(out), rs, (int32_t)rows, (int32_t)cols, (int32_t)kind, (float)c0, (float)c1,
                             dtype_of(in, "activate_rows: in"), d.stream()),
             "tah_activate_rows");
    return out;
}

void conv_rows(const Tensor& h, const InputConv& conv, const Portions& p, const Tensor& out) {
    need_lib();
    Dev d; d.see(h); d.see(out); d.see(conv.w); d.see(conv.state);
    const tah_portions P = p.c(d);
    const int64_t cols = conv.w.size(1);
    flat(h, conv.state.scalar_type(), P.rows * cols, "conv_rows: h"); flat(out, conv.state.scalar_type(), P.rows * cols, "conv_rows: out");
    check_rc(g.conv_rows(ptr(h), at_<float>(conv.w), mptr(conv.state), &P, mptr(out), (int32_t)cols, (int32_t)conv.w.size(0), (int32_t)conv.state.size(0),
                         dtype_of(h, "conv_rows: h"), d.stream()),
             "tah_conv_rows");
}

// One gated delta-rule layer: its constants, small weights and state.
struct DeltaLayer {
    Tensor conv, a_log, dt_bias, norm, conv_state, state;
    tah_delta_layer L{};
    int64_t proj_cols = 0;
    DeltaLayer(Tensor conv_, Tensor a_log_, Tensor dt_bias_, Tensor norm_, Tensor conv_state_, Tensor state_, int64_t heads, int64_t kv_heads,
               int64_t dim, int64_t vdim, std::vector<int64_t> cols, double eps)
        : conv(conv_), a_log(a_log_), dt_bias(dt_bias_), norm(norm_), conv_state(conv_state_), state(state_) {
        TORCH_CHECK(cols.size() == 6, "DeltaLayer: six column offsets (q, k, v, gate, b, a)");
        TORCH_CHECK(heads > 0 && kv_heads > 0 && dim > 0 && vdim > 0 && heads % kv_heads == 0, "DeltaLayer: heads and sizes");
        const int64_t nch = 2 * kv_heads * dim + heads * vdim;
        TORCH_CHECK(conv.dim() == 2 && conv_state.dim() == 3 && state.dim() == 4, "DeltaLayer: conv [channels, taps], conv_state [slots, taps, channels], "
                    "state [slots, heads, dim, vdim]");
        L.taps = (int32_t)conv.size(1); L.nslots = (int32_t)state.size(0);
        flat(conv, at::kFloat, nch * L.taps, "DeltaLayer: conv");
        flat(a_log, at::kFloat, heads, "DeltaLayer: a_log"); flat(dt_bias, at::kFloat, heads, "DeltaLayer: dt_bias");
        flat(norm, at::kFloat, vdim, "DeltaLayer: norm");
        L.dtype = dtype_of(conv_state, "DeltaLayer: conv_state");
        flat(conv_state, conv_state.scalar_type(), (int64_t)L.nslots * L.taps * nch, "DeltaLayer: conv_state");
        flat(state, at::kFloat, (int64_t)L.nslots * heads * dim * vdim, "DeltaLayer: state");
        L.conv = at_<float>(conv); L.a_log = at_<float>(a_log); L.dt_bias = at_<float>(dt_bias); L.norm = at_<float>(norm);
        L.conv_state = mptr(conv_state); L.state = at_<float>(state);
        L.heads = (int32_t)heads; L.kv_heads = (int32_t)kv_heads; L.dim = (int32_t)dim; L.vdim = (int32_t)vdim; L.eps = (float)eps;
        L.q_col = (int32_t)cols[0]; L.k_col = (int32_t)cols[1]; L.v_col = (int32_t)cols[2];
        L.gate_col = (int32_t)cols[3]; L.b_col = (int32_t)cols[4]; L.a_col = (int32_t)cols[5];
        const int64_t ends[] = {cols[0] + kv_heads * dim, cols[1] + kv_heads * dim, cols[2] + heads * vdim, cols[3] + heads * vdim, cols[4] + heads,
                                cols[5] + heads};
        for (int64_t e : ends) proj_cols = e > proj_cols ? e : proj_cols;
        for (int64_t c : cols) TORCH_CHECK(c >= 0, "DeltaLayer: a negative column");
    }
    tah_delta_layer with(Dev& d, const Tensor& proj, int64_t rows) const {
        d.see(proj); d.see(state); d.see(conv);
        tah_delta_layer l = L;
        l.proj_row_stride = matrix(proj, elem_type(L.dtype), rows, proj_cols, "DeltaLayer: proj");
        l.proj = ptr(proj);
        return l;
    }
    void step(const Tensor& proj, const Tensor& slot, const Tensor& pos, const optional<Tensor>& out, const optional<Tensor>& out_packed) const {
        need_lib();
        const int64_t rows = slot.numel();
        Dev d; d.see(slot); d.see(pos); d.see(out); d.see(out_packed);
        const tah_delta_layer l = with(d, proj, rows);
        flat(slot, at::kInt, rows, "DeltaLayer.step: slot"); flat(pos, at::kInt, rows, "DeltaLayer.step: pos");
        TORCH_CHECK(out.has_value() || out_packed.has_value(), "DeltaLayer.step: nothing to write");
        int64_t rs = 0, cols = 0;
        if (out.has_value()) { cols = out->size(1); rs = matrix(*out, elem_type(L.dtype), rows, cols, "DeltaLayer.step: out"); }
        if (out_packed.has_value()) {
            flat(*out_packed, at::kBFloat16, -1, "DeltaLayer.step: out_packed");
            TORCH_CHECK(out_packed->numel() % 1024 == 0 && (cols == 0 || cols == out_packed->numel() / 32), "DeltaLayer.step: out_packed must hold 32 * cols elements");
            cols = out_packed->numel() / 32;
        }
        check_rc(g.delta_step(&l, at_<int32_t>(slot), at_<int32_t>(pos), (int32_t)rows, any(out), rs, any(out_packed), (int32_t)cols, d.stream()),
                 "tah_delta_step");
    }
    // conv, recurrence, norm and gate of a batch of portions -> out [rows, cols]
    void portions(const Tensor& proj, const Portions& p, const Tensor& out) const {
        need_lib();
        Dev d;
        const tah_portions P = p.c(d);
        const tah_delta_layer l = with(d, proj, P.rows);
        d.see(out);
        const int64_t rs = matrix(out, elem_type(L.dtype), P.rows, (int64_t)L.heads * L.vdim, "DeltaLayer.portions: out");
        const auto f32 = proj.options().dtype(at::kFloat);
        Tensor q = at::empty({P.rows, L.kv_heads, L.dim}, f32), k = at::empty_like(q), v = at::empty({P.rows, L.heads, L.vdim}, f32);
        Tensor lg = at::empty({P.rows, L.heads}, f32), beta = at::empty_like(lg), o = at::empty_like(v);
        check_rc(g.delta_prepare(&l, &P, at_<float>(q), at_<float>(k), at_<float>(v), at_<float>(lg), at_<float>(beta), d.stream()), "tah_delta_prepare");
        const size_t bytes = g.delta_scan_workspace(&l, P.nseq, P.rows);
        Tensor work = at::empty({(int64_t)bytes}, proj.options().dtype(at::kByte));
        check_rc(g.delta_scan(&l, &P, at_<float>(q), at_<float>(k), at_<float>(v), at_<float>(lg), at_<float>(beta), at_<float>(o), mptr(work), bytes,
                              d.stream()),
                 "tah_delta_scan");
        check_rc(g.delta_finish(&l, at_<float>(o), P.rows, mptr(out), rs, (int32_t)out.size(1), d.stream()), "tah_delta_finish");
    }
};

// One latent-attention layer on a ring of cached rows (its own or another layer's).
struct LatentLayer {
    Tensor ring;
    tah_latent_layer L{};
    LatentLayer(Tensor ring_, int64_t heads, int64_t dim_pad, int64_t rot_dim, int64_t rot_pad, int64_t rank, int64_t rank_pad, int64_t vdim_pad,
                int64_t window, double scale)
        : ring(ring_) {
        TORCH_CHECK(ring.dim() == 3 && ring.is_contiguous() && ring.size(2) == rank_pad + rot_pad, "LatentLayer: ring [slots, capacity, rank_pad + rot_pad]");
        L.dtype = dtype_of(ring, "LatentLayer: ring");
        L.ring = mptr(ring);
        L.heads = (int32_t)heads; L.dim_pad = (int32_t)dim_pad; L.rot_dim = (int32_t)rot_dim; L.rot_pad = (int32_t)rot_pad; L.rank = (int32_t)rank;
        L.rank_pad = (int32_t)rank_pad; L.vdim_pad = (int32_t)vdim_pad; L.capacity = (int32_t)ring.size(1); L.nslots = (int32_t)ring.size(0);
        L.window = (int32_t)window; L.scale = (float)scale;
    }
    int64_t row() const { return L.rank_pad + L.rot_pad; }
    void prep(const Tensor& proj, int64_t q_col, int64_t dkv_col, const optional<Tensor>& norm, double eps, const Tensor& cos, const Tensor& sin,
              const Tensor& pos, const optional<Tensor>& slot, const optional<Tensor>& rows_out, const optional<Tensor>& q_packed,
              const optional<Tensor>& q_rows) const {
        need_lib();
        Dev d; d.see(ring); d.see(proj); d.see(norm); d.see(cos); d.see(sin); d.see(pos); d.see(slot); d.see(rows_out); d.see(q_packed); d.see(q_rows);
        const int64_t rows = pos.numel(), hq = (int64_t)L.heads * (L.dim_pad + L.rot_pad);
        const at::ScalarType ty = elem_type(L.dtype);
        tah_latent_prep_args a{};
        int64_t need = q_col + hq;
        if (dkv_col >= 0 && dkv_col + L.rank + L.rot_dim > need) need = dkv_col + L.rank + L.rot_dim;
        a.proj_row_stride = matrix(proj, ty, rows, need, "LatentLayer.prep: proj");
        a.proj = mptr(proj);
        a.q_col = (int32_t)q_col; a.dkv_col = (int32_t)dkv_col;
        flat(pos, at::kInt, rows, "LatentLayer.prep: pos"); flat(slot, at::kInt, rows, "LatentLayer.prep: slot");
        flat(norm, at::kFloat, L.rank, "LatentLayer.prep: norm");
        TORCH_CHECK(dkv_col < 0 || norm.has_value(), "LatentLayer.prep: the latent's norm is missing");
        TORCH_CHECK(cos.dim() == 2 && cos.size(1) == L.rot_dim / 2, "LatentLayer.prep: cos / sin must be [positions, rot_dim / 2]");
        flat(cos, at::kFloat, -1, "LatentLayer.prep: cos"); flat(sin, at::kFloat, cos.numel(), "LatentLayer.prep: sin");
        flat(rows_out, ty, rows * row(), "LatentLayer.prep: rows_out");
        flat(q_packed, at::kBFloat16, (int64_t)L.heads * 32 * L.dim_pad, "LatentLayer.prep: q_packed");
        flat(q_rows, ty, (int64_t)L.heads * rows * L.dim_pad, "LatentLayer.prep: q_rows");
        a.norm = at_<float>(norm); a.cos = at_<float>(cos); a.sin = at_<float>(sin); a.pos = at_<int32_t>(pos); a.slot = at_<int32_t>(slot);
        a.rows_out = any(rows_out); a.q_packed = any(q_packed); a.q_rows = any(q_rows);
        a.rows = (int32_t)rows; a.table_rows = (int32_t)cos.size(0); a.eps = (float)eps;
        check_rc(g.latent_prep(&L, &a, d.stream()), "tah_latent_prep");
    }
    void context(const Portions& p, const Tensor& cu_k, const Tensor& new_rows, const Tensor& ctx) const {
        need_lib();
        Dev d; d.see(ring); d.see(cu_k); d.see(new_rows); d.see(ctx);
        const tah_portions P = p.c(d);
        flat(cu_k, at::kInt, P.nseq + 1, "LatentLayer.context: cu_k");
        flat(new_rows, elem_type(L.dtype), P.rows * row(), "LatentLayer.context: new_rows");
        TORCH_CHECK(ctx.dim() == 2 && ctx.size(1) == row(), "LatentLayer.context: ctx must be [rows, rank_pad + rot_pad]");
        flat(ctx, elem_type(L.dtype), -1, "LatentLayer.context: ctx");
        check_rc(g.latent_context(&L, &P, at_<int32_t>(cu_k), (int32_t)ctx.size(0), ptr(new_rows), mptr(ctx), d.stream()), "tah_latent_context");
    }
    void attend(const Portions& p, const Tensor& cu_k, int64_t max_rows, const Tensor& proj, int64_t q_col, const Tensor& k, const Tensor& v,
                const Tensor& ctx, const Tensor& out) const {
        need_lib();
        Dev d; d.see(cu_k); d.see(proj); d.see(k); d.see(v); d.see(ctx); d.see(out);
        const tah_portions P = p.c(d);
        const at::ScalarType ty = elem_type(L.dtype);
        const int64_t n = ctx.size(0), hq = (int64_t)L.heads * (L.dim_pad + L.rot_pad);
        flat(cu_k, at::kInt, P.nseq + 1, "LatentLayer.attend: cu_k");
        const int64_t qs = matrix(proj, ty, P.rows, q_col + hq, "LatentLayer.attend: proj");
        const int64_t ks = matrix(k, ty, n, (int64_t)L.heads * L.dim_pad, "LatentLayer.attend: k");
        const int64_t vs = matrix(v, ty, n, (int64_t)L.heads * L.vdim_pad, "LatentLayer.attend: v");
        TORCH_CHECK(ctx.dim() == 2 && ctx.size(1) == row(), "LatentLayer.attend: ctx must be [rows, rank_pad + rot_pad]");
        flat(ctx, ty, -1, "LatentLayer.attend: ctx");
        const int64_t os = matrix(out, ty, P.rows, (int64_t)L.heads * L.vdim_pad, "LatentLayer.attend: out");
        check_rc(g.latent_attend(&L, &P, at_<int32_t>(cu_k), (int32_t)max_rows,
                                 static_cast<const char*>(ptr(proj)) + q_col * proj.element_size(), qs, ptr(k), ks, ptr(v), vs, ptr(ctx), mptr(out), os,
                                 d.stream()),
                 "tah_latent_attend");
    }
    int64_t decode_workspace(int64_t rows) const { need_lib(); return (int64_t)g.latent_decode_workspace(&L, (int32_t)rows); }
    void decode(const Tensor& slot, const Tensor& pos, const Tensor& q_latent, const Tensor& proj, int64_t q_col, const optional<Tensor>& out_packed,
                const optional<Tensor>& out_rows, const optional<Tensor>& workspace) const {
        need_lib();
        Dev d; d.see(ring); d.see(slot); d.see(pos); d.see(q_latent); d.see(proj); d.see(out_packed); d.see(out_rows); d.see(workspace);
        const int64_t rows = slot.numel(), hq = (int64_t)L.heads * (L.dim_pad + L.rot_pad);
        const at::ScalarType ty = elem_type(L.dtype);
        flat(slot, at::kInt, rows, "LatentLayer.decode: slot"); flat(pos, at::kInt, rows, "LatentLayer.decode: pos");
        flat(q_latent, ty, (int64_t)L.heads * rows * L.rank_pad, "LatentLayer.decode: q_latent");
        const int64_t qs = matrix(proj, ty, rows, q_col + hq, "LatentLayer.decode: proj");
        flat(out_packed, at::kBFloat16, (int64_t)L.heads * 32 * L.rank_pad, "LatentLayer.decode: out_packed");
        flat(out_rows, ty, (int64_t)L.heads * rows * L.rank_pad, "LatentLayer.decode: out_rows");
        flat(workspace, at::kByte, -1, "LatentLayer.decode: workspace");
        check_rc(g.latent_decode(&L, at_<int32_t>(slot), at_<int32_t>(pos), (int32_t)rows, ptr(q_latent), rows * L.rank_pad,
                                 static_cast<const char*>(ptr(proj)) + q_col * proj.element_size(), qs, any(out_packed), any(out_rows), any(workspace),
                                 workspace.has_value() ? (size_t)workspace->numel() : 0, d.stream()),
                 "tah_latent_decode");
    }
};

// One layer of attention in a window with kept first tokens, on a cache of rows [slots, kv_heads, keep + ring, row].
struct WindowLayer {
    Tensor cache, cos, sin;
    tah_window_layer L{};
    int64_t q_col, k_col, g_col;
    WindowLayer(Tensor cache_, Tensor cos_, Tensor sin_, int64_t heads, int64_t key_dim, int64_t value_dim, int64_t rot_dim, int64_t rot_pad,
                int64_t rot_source, int64_t keep_first, int64_t window, double scale, int64_t q_col_, int64_t k_col_, int64_t g_col_)
        : cache(cache_), cos(cos_), sin(sin_), q_col(q_col_), k_col(k_col_), g_col(g_col_) {
        TORCH_CHECK(cache.dim() == 4 && cache.is_contiguous() && keep_first >= 0 && cache.size(2) > keep_first,
                    "WindowLayer: cache [slots, kv_heads, keep_first + ring, row]");
        TORCH_CHECK(cos.dim() == 2 && cos.size(1) == rot_dim / 2, "WindowLayer: cos / sin must be [positions, rot_dim / 2]");
        flat(cos, at::kFloat, -1, "WindowLayer: cos"); flat(sin, at::kFloat, cos.numel(), "WindowLayer: sin");
        L.dtype = dtype_of(cache, "WindowLayer: cache");
        L.cache = mptr(cache);
        L.heads = (int32_t)heads; L.kv_heads = (int32_t)cache.size(1); L.row = (int32_t)cache.size(3); L.key_dim = (int32_t)key_dim;
        L.value_dim = (int32_t)value_dim; L.rot_dim = (int32_t)rot_dim; L.rot_pad = (int32_t)rot_pad; L.rot_source = (int32_t)rot_source;
        L.keep_first = (int32_t)keep_first; L.ring = (int32_t)(cache.size(2) - keep_first); L.window = (int32_t)window; L.nslots = (int32_t)cache.size(0);
        L.scale = (float)scale;
    }
    tah_window_rows rows(Dev& d, const Tensor& proj, const Tensor& pos, const optional<Tensor>& slot) const {
        d.see(cache); d.see(cos); d.see(sin); d.see(proj); d.see(pos); d.see(slot);
        const int64_t n = pos.numel();
        int64_t need = std::max(q_col + (int64_t)L.heads * L.key_dim, k_col + (int64_t)L.kv_heads * L.row);
        if (g_col >= 0) need = std::max(need, g_col + L.heads);
        flat(pos, at::kInt, n, "WindowLayer: pos"); flat(slot, at::kInt, n, "WindowLayer: slot");
        tah_window_rows r{};
        r.proj_row_stride = matrix(proj, elem_type(L.dtype), n, need, "WindowLayer: proj");
        r.proj = mptr(proj); r.cos = at_<float>(cos); r.sin = at_<float>(sin); r.pos = at_<int32_t>(pos); r.slot = at_<int32_t>(slot);
        r.q_col = (int32_t)q_col; r.k_col = (int32_t)k_col; r.g_col = (int32_t)g_col; r.rows = (int32_t)n; r.table_rows = (int32_t)cos.size(0);
        return r;
    }
    int64_t width() const { return (int64_t)L.heads * L.value_dim; }
    // rotation, attention and cache of a batch of portions -> out [rows, >= heads * value_dim]; proj is rotated in place
    void portions(const Tensor& proj, const Portions& p, const Tensor& pos, const Tensor& out) const {
        need_lib();
        Dev d; d.see(out);
        const tah_window_rows r = rows(d, proj, pos, c10::nullopt);
        const tah_portions P = p.c(d);
        const int64_t rs = matrix(out, elem_type(L.dtype), r.rows, width(), "WindowLayer.portions: out");
        check_rc(g.window_prep(&L, &r, d.stream()), "tah_window_prep");
        check_rc(g.window_attend(&L, &P, &r, mptr(out), rs, d.stream()), "tah_window_attend");
        check_rc(g.window_append(&L, &P, &r, d.stream()), "tah_window_append");
    }
    int64_t decode_workspace(int64_t n) const { need_lib(); return (int64_t)g.window_decode_workspace(&L, (int32_t)n); }
    void decode(const Tensor& proj, const Tensor& slot, const Tensor& pos, const optional<Tensor>& out, const optional<Tensor>& out_packed,
                const optional<Tensor>& workspace) const {
        need_lib();
        Dev d; d.see(out); d.see(out_packed); d.see(workspace);
        const tah_window_rows r = rows(d, proj, pos, slot);
        const int64_t rs = out.has_value() ? matrix(*out, elem_type(L.dtype), r.rows, width(), "WindowLayer.decode: out") : 0;
        flat(out_packed, at::kBFloat16, 32 * width(), "WindowLayer.decode: out_packed");
        flat(workspace, at::kByte, -1, "WindowLayer.decode: workspace");
        check_rc(g.window_decode(&L, &r, any(out), rs, any(out_packed), any(workspace), workspace.has_value() ? (size_t)workspace->numel() : 0, d.stream()),
                 "tah_window_decode");
    }
};

void moe_route(const Tensor& x, const Tensor& router, const optional<Tensor>& gate_w, const Tensor& index, const Tensor& weight,
               const optional<Tensor>& shared_gate, int64_t score, int64_t groups, int64_t keep) {
    need_lib();
    Dev d; d.see(x); d.see(router); d.see(gate_w); d.see(index); d.see(weight); d.see(shared_gate);
    TORCH_CHECK(x.dim() == 2 && router.dim() == 2 && router.size(1) == x.size(1) && index.dim() == 2, "moe_route: x [rows, cols], router [experts, cols]");
    const int64_t rows = x.size(0), cols = x.size(1), top = index.size(1);
    const bool x_elem = x.scalar_type() == router.scalar_type();
    flat(x, x_elem ? router.scalar_type() : at::kFloat, rows * cols, "moe_route: x"); flat(router, router.scalar_type(), -1, "moe_route: router");
    flat(gate_w, router.scalar_type(), cols, "moe_route: gate_w"); flat(index, at::kInt, rows * top, "moe_route: index");
    flat(weight, at::kFloat, rows * top, "moe_route: weight"); flat(shared_gate, at::kFloat, rows, "moe_route: shared_gate");
    TORCH_CHECK(gate_w.has_value() == shared_gate.has_value(), "moe_route: gate_w and shared_gate come together");
    const tah_moe_route_args a{ptr(x), ptr(router), any(gate_w), at_<int32_t>(index), at_<float>(weight), at_<float>(shared_gate), (int32_t)rows,
                               (int32_t)cols, (int32_t)router.size(0), (int32_t)top, (int32_t)groups, (int32_t)keep, (int32_t)score, x_elem,
                               dtype_of(router, "moe_route: router")};
    check_rc(g.moe_route(&a, d.stream()), "tah_moe_route");
}

// -> source [places], tile_expert [tiles and their number], place [rows, top]
std::vector<Tensor> moe_plan(const Tensor& index, int64_t experts) {
    need_lib();
    Dev d; d.see(index);
    TORCH_CHECK(index.dim() == 2, "moe_plan: index must be [rows, top]");
    flat(index, at::kInt, -1, "moe_plan: index");
    const int64_t rows = index.size(0), top = index.size(1);
    const int64_t places = g.moe_places((int32_t)rows, (int32_t)top, (int32_t)experts);
    Tensor source = at::empty({places}, index.options()), tile = at::empty({places / TAH_MOE_TILE + 1}, index.options()), place = at::empty_like(index);
    check_rc(g.moe_plan(at_<int32_t>(index), (int32_t)rows, (int32_t)top, (int32_t)experts, at_<int32_t>(source), at_<int32_t>(tile), at_<int32_t>(place),
                        d.stream()),
             "tah_moe_plan");
    return {source, tile, place};
}

Tensor moe_linear(const Tensor& x, const Tensor& w, const Tensor& source, const Tensor& tile_expert, bool gate_up, bool clamped, double c0, double c1) {
    need_lib();
    Dev d; d.see(x); d.see(w); d.see(source); d.see(tile_expert);
    TORCH_CHECK(w.dim() == 3 && w.is_contiguous() && (!gate_up || w.size(1) % 2 == 0), "moe_linear: w must be a contiguous [experts, n, k] tensor");
    const int64_t n = gate_up ? w.size(1) / 2 : w.size(1), k = w.size(2), tiles = tile_expert.numel() - 1;
    flat(tile_expert, at::kInt, -1, "moe_linear: tile_expert"); flat(source, at::kInt, tiles * TAH_MOE_TILE, "moe_linear: source");
    const int64_t rs = matrix(x, w.scalar_type(), gate_up ? 1 : tiles * TAH_MOE_TILE, k, "moe_linear: x");
    Tensor out = at::empty({tiles * TAH_MOE_TILE, n}, x.options());
    check_rc(g.moe_linear(ptr(x), rs, ptr(w), at_<int32_t>(source), at_<int32_t>(tile_expert), (int32_t)tiles, (int32_t)n, (int32_t)k,
                          gate_up ? TAH_LINEAR_GATE_UP : TAH_LINEAR_PLAIN, clamped ? TAH_ACT_CLAMPED_GATE : TAH_ACT_NONE, (float)c0, (float)c1, mptr(out), n, dtype_of(w, "moe_linear: w"), d.stream()),
             "tah_moe_linear");
    return out;
}

}  // namespace

void bind_mixers(py::module_& m) {
    m.def("embed_rows", &embed_rows);
    py::class_<InputConv>(m, "InputConv").def(py::init<Tensor, Tensor>());
    m.def("residual_norm", &residual_norm);
    m.def("conv_rows", &conv_rows);
    m.def("activate_rows", &activate_rows);
    m.def("moe_route", &moe_route);
    m.def("moe_plan", &moe_plan);
    m.def("moe_linear", &moe_linear);
    py::class_<Portions>(m, "Portions").def(py::init<Tensor, Tensor, Tensor, Tensor>());
    py::class_<DeltaLayer>(m, "DeltaLayer")
        .def(py::init<Tensor, Tensor, Tensor, Tensor, Tensor, Tensor, int64_t, int64_t, int64_t, int64_t, std::vector<int64_t>, double>())
        .def("step", &DeltaLayer::step)
        .def("portions", &DeltaLayer::portions);
    py::class_<LatentLayer>(m, "LatentLayer")
        .def(py::init<Tensor, int64_t, int64_t, int64_t, int64_t, int64_t, int64_t, int64_t, int64_t, double>())
        .def("prep", &LatentLayer::prep)
        .def("context", &LatentLayer::context)
        .def("attend", &LatentLayer::attend)
        .def("decode_workspace", &LatentLayer::decode_workspace)
        .def("decode", &LatentLayer::decode);
    py::class_<WindowLayer>(m, "WindowLayer")
        .def(py::init<Tensor, Tensor, Tensor, int64_t, int64_t, int64_t, int64_t, int64_t, int64_t, int64_t, int64_t, double, int64_t, int64_t, int64_t>())
        .def("portions", &WindowLayer::portions)
        .def("decode_workspace", &WindowLayer::decode_workspace)
        .def("decode", &WindowLayer::decode);
}

}  // namespace tah_ext
