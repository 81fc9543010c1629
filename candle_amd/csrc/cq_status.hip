// Text of the status codes, in a file of its own: both libraries carry it.
#include "cq_device.h"

extern "C" {

const char *cq_status_string(int status) {
    switch (status) {
        case CQ_OK: return "ok";
        case CQ_ERR_DTYPE: return "dtype not supported by this entry point";
        case CQ_ERR_SHAPE: return "invalid shape (k must be a positive multiple of the block size, sizes must be non-negative)";
        case CQ_ERR_ALIGN: return "pointer alignment requirement not met";
        case CQ_ERR_NULL: return "required pointer is NULL";
        case CQ_ERR_WORKSPACE: return "workspace too small";
        case CQ_ERR_RANGE: return "size exceeds what this entry point supports";
    }
    if (status > 0) return hipGetErrorString((hipError_t)status);
    return "unknown status";
}

}  // extern "C"
