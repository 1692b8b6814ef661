#include "device_util.h"
#include "stack_ops.h"
namespace mimir {
hipError_t gemm_bf16(const uint16_t* W, int64_t ldw, const uint16_t* x, int64_t ldx, int64_t M, int64_t N, int64_t K, const ProductOut& out, hipStream_t st) { return hipErrorNotSupported; }
}
