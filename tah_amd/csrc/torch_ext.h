// Shared by the translation units of the PyTorch-ROCm extension: the entry points of the loaded library, and what every
// binding needs to turn tensors into the C ABI's arguments.
#pragma once
#include <c10/hip/HIPStream.h>
#include <torch/extension.h>

#include <string>

#include "tah_duo.h"
#include "tah_mixers.h"

namespace tah_ext {

using at::Tensor;
using c10::optional;

// An entry point of the loaded library; a library that holds only some of the kernels leaves the others empty.
template <class F>
struct Entry;
template <class R, class... A>
struct Entry<R (*)(A...)> {
    R (*f)(A...) = nullptr;
    const char* name = "";
    R operator()(A... a) const {
        TORCH_CHECK(f != nullptr, "tah_amd: ", name, " is not part of the loaded library (build the whole of it: make -C tah_amd/csrc)");
        return f(a...);
    }
};

struct Api {
    void* handle = nullptr;
    bool allow_host = false;
    Entry<decltype(&tah_duo_abi_version)> abi_version;
    Entry<decltype(&tah_duo_error_string)> error_string;
    Entry<decltype(&tah_duo_fwd_varlen)> fwd_varlen;
    Entry<decltype(&tah_duo_bwd_varlen)> bwd_varlen;
    Entry<decltype(&tah_duo_bwd_workspace_bytes)> bwd_workspace_bytes;
    Entry<decltype(&tah_duo_schedule_bytes)> schedule_bytes;
    Entry<decltype(&tah_duo_schedule_build)> schedule_build;
    Entry<decltype(&tah_greedy_step)> greedy_step;
    Entry<decltype(&tah_silu_mul_normed)> silu_mul_normed;
    Entry<decltype(&tah_step_begin)> step_begin;
    Entry<decltype(&tah_greedy_tick)> greedy_tick;
    Entry<decltype(&tah_decider_tail)> decider_tail;
    Entry<decltype(&tah_linear_pack_weight)> linear_pack_weight;
    Entry<decltype(&tah_linear_pack_rows)> linear_pack_rows;
    Entry<decltype(&tah_linear_rows)> linear_rows;
    Entry<decltype(&tah_duo_fwd_masked)> fwd_masked;
    Entry<decltype(&tah_duo_bwd_masked)> bwd_masked;
    Entry<decltype(&tah_duo_decode_workspace_bytes)> decode_workspace_bytes;
    Entry<decltype(&tah_duo_decode)> decode;
    Entry<decltype(&tah_duo_decode_static)> decode_static;
    Entry<decltype(&tah_kv_append)> kv_append;
    Entry<decltype(&tah_qk_prep)> qk_prep;
    Entry<decltype(&tah_duo_decode_step)> decode_step;
    Entry<decltype(&tah_duo_decode_step_supported)> decode_step_supported;
    Entry<decltype(&tah_topk_mix)> topk_mix;
    Entry<decltype(&tah_qk_prep_bwd)> qk_prep_bwd;
    Entry<decltype(&tah_sample_rows)> sample_rows;
    Entry<decltype(&tah_silu_mul)> silu_mul;
    Entry<decltype(&tah_hard_index_build)> hard_index_build;
    Entry<decltype(&tah_pad_rows_build)> pad_rows_build;
    Entry<decltype(&tah_rows_copy)> rows_copy;
    Entry<decltype(&tah_embed_rows)> embed_rows;
    Entry<decltype(&tah_residual_norm)> residual_norm;
    Entry<decltype(&tah_activate_rows)> activate_rows;
    Entry<decltype(&tah_conv_rows)> conv_rows;
    Entry<decltype(&tah_delta_step)> delta_step;
    Entry<decltype(&tah_delta_prepare)> delta_prepare;
    Entry<decltype(&tah_delta_scan)> delta_scan;
    Entry<decltype(&tah_delta_scan_workspace)> delta_scan_workspace;
    Entry<decltype(&tah_delta_finish)> delta_finish;
    Entry<decltype(&tah_latent_prep)> latent_prep;
    Entry<decltype(&tah_latent_context)> latent_context;
    Entry<decltype(&tah_latent_attend)> latent_attend;
    Entry<decltype(&tah_latent_decode_workspace)> latent_decode_workspace;
    Entry<decltype(&tah_latent_decode)> latent_decode;
    Entry<decltype(&tah_window_prep)> window_prep;
    Entry<decltype(&tah_window_attend)> window_attend;
    Entry<decltype(&tah_window_append)> window_append;
    Entry<decltype(&tah_window_decode_workspace)> window_decode_workspace;
    Entry<decltype(&tah_window_decode)> window_decode;
    Entry<decltype(&tah_moe_route)> moe_route;
    Entry<decltype(&tah_moe_places)> moe_places;
    Entry<decltype(&tah_moe_plan)> moe_plan;
    Entry<decltype(&tah_moe_linear)> moe_linear;
};
extern Api g;

inline void need_lib() { TORCH_CHECK(g.handle != nullptr, "tah_amd: no library loaded (tah_amd._lib.lib() loads libtah_duo.so)"); }

inline void check_rc(int rc, const char* what) {
    TORCH_CHECK(rc == 0, what, ": ", g.error_string(rc), " (code ", rc, ")");
}

// One device for all tensors; host tensors only when the loaded library is the host build of the kernels.
struct Dev {
    bool set = false;
    c10::Device dev{c10::kCPU};
    void see(const Tensor& t) {
        if (!t.defined()) return;
        TORCH_CHECK(t.is_cuda() || g.allow_host, "tah_amd ops need CUDA/HIP tensors (no CPU path exists)");
        if (!set) { dev = t.device(); set = true; }
        else TORCH_CHECK(t.device() == dev, "tensors on different devices: ", dev, " vs ", t.device());
    }
    void see(const optional<Tensor>& t) { if (t.has_value()) see(*t); }
    tah_stream_t stream() const {
        if (set && dev.is_cuda()) return static_cast<tah_stream_t>(c10::hip::getCurrentHIPStream(dev.index()).stream());
        return nullptr;
    }
};

inline const void* ptr(const Tensor& t) { return (!t.defined() || t.numel() == 0) ? nullptr : t.data_ptr(); }
inline void* mptr(const Tensor& t) { return (!t.defined() || t.numel() == 0) ? nullptr : t.data_ptr(); }
inline const void* ptr(const optional<Tensor>& t) { return t.has_value() ? ptr(*t) : nullptr; }

void bind_mixers(pybind11::module_& m);

}  // namespace tah_ext
