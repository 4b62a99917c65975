// abi_core.hip -- the part of include/bitnet_hip.h every model needs: lifecycle, error text, device information, position and
// greedy-token operators.
#include <cstring>
#include <mutex>
#include <vector>

#include "common.hpp"

namespace bitnet_hip {

thread_local std::string g_last_error;
int g_device = 0;

namespace {
std::mutex g_mu;
bool g_inited = false;
std::vector<void (*)()> &cleanups() {
    static std::vector<void (*)()> v;
    return v;
}
}  // namespace

void at_cleanup(void (*fn)()) { cleanups().push_back(fn); }

int ensure_init() {
    {
        std::lock_guard<std::mutex> lk(g_mu);
        if (g_inited) return BITNET_HIP_OK;
    }
    return bitnet_hip_init(-1);
}

}  // namespace bitnet_hip

using namespace bitnet_hip;

extern "C" {

int bitnet_hip_init(int device) {
    BH_GUARD_BEGIN
    int count = 0;
    hipError_t e = hipGetDeviceCount(&count);
    if (e != hipSuccess || count <= 0)
        return set_error(BITNET_HIP_ERR_GPU, "no HIP device available (hipGetDeviceCount: %s)",
                         hipGetErrorString(e));
    if (device < 0) {
        if (hipGetDevice(&device) != hipSuccess) device = 0;
    }
    if (device >= count)
        return set_error(BITNET_HIP_ERR_INVALID_ARGUMENT, "device %d out of range (%d visible)", device,
                         count);
    BH_HIP_TRY(hipSetDevice(device));
    hipDeviceProp_t prop;
    BH_HIP_TRY(hipGetDeviceProperties(&prop, device));
    if (strncmp(prop.gcnArchName, "gfx950", 6) != 0)
        return set_error(BITNET_HIP_ERR_UNSUPPORTED,
                         "device %d is %s; this library carries gfx950 (MI355X) code objects only",
                         device, prop.gcnArchName);
    std::lock_guard<std::mutex> lk(g_mu);
    g_device = device;
    g_inited = true;
    g_last_error.clear();
    return BITNET_HIP_OK;
    BH_GUARD_END
}

void bitnet_hip_cleanup(void) {
    try {
        for (void (*fn)() : cleanups()) fn();
        std::lock_guard<std::mutex> lk(g_mu);
        g_inited = false;
        g_last_error.clear();
    } catch (...) {
    }
}

int bitnet_hip_is_available(void) {
    int count = 0;
    return hipGetDeviceCount(&count) == hipSuccess && count > 0 ? 1 : 0;
}

int bitnet_hip_device_count(void) {
    int count = 0;
    return hipGetDeviceCount(&count) == hipSuccess ? count : 0;
}

const char *bitnet_hip_get_last_error(void) {
    return g_last_error.empty() ? nullptr : g_last_error.c_str();
}

int bitnet_hip_get_device_info(int device, bitnet_hip_device_info *out) {
    BH_GUARD_BEGIN
    if (!out) return set_error(BITNET_HIP_ERR_INVALID_ARGUMENT, "Null pointer passed to get_device_info");
    hipDeviceProp_t prop;
    BH_HIP_TRY(hipGetDeviceProperties(&prop, device));
    memset(out, 0, sizeof(*out));
    out->device_id = device;
    strncpy(out->name, prop.name, sizeof(out->name) - 1);
    strncpy(out->gcn_arch, prop.gcnArchName, sizeof(out->gcn_arch) - 1);
    out->total_memory = prop.totalGlobalMem;
    out->compute_unit_count = prop.multiProcessorCount;
    out->max_wavefront_size = prop.warpSize;
    out->max_shared_memory_per_workgroup = prop.sharedMemPerBlock;
    out->supports_fp16 = 1;
    out->supports_bf16 = 1;
    return BITNET_HIP_OK;
    BH_GUARD_END
}

int bitnet_hip_advance_pos_dev(int32_t *pos_dev, void *stream) {
    BH_GUARD_BEGIN
    if (!pos_dev) return set_error(BITNET_HIP_ERR_INVALID_ARGUMENT, "Null pointer passed to advance_pos_dev");
    BH_HIP_TRY(launch_advance_pos(pos_dev, (hipStream_t)stream));
    return BITNET_HIP_OK;
    BH_GUARD_END
}

int bitnet_hip_argmax_dev(const float *v, size_t n, void *scratch, size_t n_wg, int32_t *token_dev, void *stream) {
    BH_GUARD_BEGIN
    if (!v || !scratch || !token_dev) return set_error(BITNET_HIP_ERR_INVALID_ARGUMENT, "Null pointer passed to argmax_dev");
    if (n == 0 || n_wg == 0) return set_error(BITNET_HIP_ERR_INVALID_ARGUMENT, "argmax: empty input");
    float *bv = static_cast<float *>(scratch);
    int *bi = reinterpret_cast<int *>(bv + n_wg);
    BH_HIP_TRY(launch_argmax(v, (int)n, bv, bi, (int)n_wg, token_dev, (hipStream_t)stream));
    return BITNET_HIP_OK;
    BH_GUARD_END
}

}  // extern "C"
