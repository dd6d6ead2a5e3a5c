#include "row_io.h"
extern "C" int mi_talking_attn_supported(int32_t, int32_t, int32_t, int32_t, int32_t, float) { return 0; }
extern "C" int64_t mi_talking_decode_workspace_bytes(int32_t, int32_t, int32_t, int32_t, int32_t, int32_t) { return 0; }
extern "C" int mi_talking_decode(const mi_talking_attn_args*, int32_t, int32_t, void*, int64_t, void*) { return -2; }
extern "C" int64_t mi_talking_prefill_workspace_bytes(int32_t, int32_t, int32_t, int32_t, int32_t) { return 0; }
extern "C" int mi_talking_prefill(const mi_talking_attn_args*, const int32_t*, int32_t, int32_t, int32_t, int32_t, void*, int64_t, void*) { return -2; }
