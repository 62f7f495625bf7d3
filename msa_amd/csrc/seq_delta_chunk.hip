#include "seq_mfma.h"
extern "C" size_t msa_seq_delta_chunked_workspace_bytes(const msa_delta_args* args, int32_t max_rows, int32_t n_seq) { return 0; }
extern "C" int msa_seq_delta_chunked(const msa_delta_args* args, const msa_seq_batch* batch, void* workspace, size_t workspace_bytes, void* stream) { return MSA_EINVAL; }
