// Token-generation weight stream, F8E4M3 weights (templates: linear_device.h).
#define MI_TRACE_EXPORT 1
#include "linear_device.h"

namespace mi {
template int launch_gemv_wd<MI_W_F8E4M3>(const LinearW&, int, int, const ProArgs&, int, const EpiArgs&, hipStream_t);
}
