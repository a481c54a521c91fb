// What every build of the library answers about itself (host code).
#include "tah_duo.h"

extern "C" int tah_duo_abi_version(void) { return TAH_DUO_ABI_VERSION; }

extern "C" const char* tah_duo_error_string(int code) {
    switch (code) {
        case TAH_OK: return "ok";
        case TAH_E_NULL: return "a required pointer is NULL";
        case TAH_E_SHAPE: return "unsupported shape (head_dim must be 128, Hq/Hkv in {1,2,4,8}, sizes >= 0)";
        case TAH_E_ALIGN: return "pointers must be 16-byte aligned and strides multiples of 8 elements";
        case TAH_E_LAUNCH: return "HIP launch failed";
        case TAH_E_WORKSPACE: return "workspace too small";
        case TAH_E_SCRATCH: return "the call needs more split-K scratch than tah_duo_decode_static holds (TAH_DUO_STATIC_SCRATCH_BYTES)";
        default: return "unknown error";
    }
}
