// Internal interface between linear_recurrence.hip and its chunk-parallel form (chunk_recurrence.hip).
#pragma once
#include <hip/hip_runtime.h>
#include "../../include/vlm_hip.h"

#define VLM_CHUNK 64              // tokens per chunk
#define VLM_CHUNK_MIN 17          // segments of at least this many tokens take the chunk-parallel form

// the raw read-outs and states of the segments of more than max_len tokens (the other segments are left alone)
__attribute__((visibility("hidden"))) int vlm_chunk_recurrence(const vlm_recurrence_args* a, int nseg, int ntok, int max_len, int dtype, hipStream_t st);
