#include "seq_common.h"
extern "C" size_t msa_seq_ssd_chunked_workspace_bytes(int32_t, int32_t, int32_t, int32_t, int32_t) { return 0; }
extern "C" int msa_seq_ssd_chunked(const void*, int64_t, const void*, int64_t, const void*, int64_t, const float*, const float*, const float*, int32_t, int32_t, int32_t, int32_t, int32_t, float*, void*, const msa_seq_batch*, void*, size_t, void*) { return MSA_EINVAL; }
