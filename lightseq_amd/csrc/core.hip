// What every model of the library needs, whatever its kernels: status and error text, device facts,
// the route epoch, small fills, and the set-up of the random-number states.
#include <atomic>
#include <mutex>
#include <string>

#include "ls_device.h"
#include "ls_launch.h"
#include "sample_common.h"

namespace lsh {

static thread_local std::string g_last_error;

int lsh_fail(int code, const char* msg) {
  g_last_error = msg ? msg : "";
  return code;
}

int lsh_check_hip(hipError_t e, const char* what) {
  if (e == hipSuccess) return LSH_OK;
  g_last_error = std::string(what ? what : "hip") + ": " + hipGetErrorName(e) + " " +
                 hipGetErrorString(e);
  return LSH_ERR_HIP;
}

int lsh_check_launch(const char* what) { return lsh_check_hip(hipGetLastError(), what); }

static std::atomic<unsigned long> g_route_epoch{0};

unsigned long route_epoch() { return g_route_epoch.load(std::memory_order_acquire); }
void route_epoch_bump() { g_route_epoch.fetch_add(1, std::memory_order_acq_rel); }

// Compute units of the current device (256 on MI355X), read once per device: the choices below
// reason in rounds of the chip -- one, two or three resident workgroups per compute unit.
int cu_count() {
  static std::mutex mu;
  static int cached[64] = {};
  int dev = 0;
  if (hipGetDevice(&dev) != hipSuccess || dev < 0 || dev >= 64) return 256;
  std::lock_guard<std::mutex> lock(mu);
  if (cached[dev] == 0) {
    int n = 0;
    if (hipDeviceGetAttribute(&n, hipDeviceAttributeMultiprocessorCount, dev) != hipSuccess || n <= 0)
      n = 256;
    cached[dev] = n;
  }
  return cached[dev];
}

// A fill kernel for the words a generation step must clear: a memset node in a captured
// graph replays wrongly on this platform, a kernel node does not.
__global__ void fill_i32_kernel(int* __restrict__ p, int value, int n) {
  const int i = blockIdx.x * blockDim.x + threadIdx.x;
  if (i < n) p[i] = value;
}
int fill_i32(int* p, int value, int n, hipStream_t s) {
  if (!p || n <= 0) return lsh_fail(LSH_ERR_INVALID, "fill_i32: bad arguments");
  fill_i32_kernel<<<(n + 255) / 256, 256, 0, s>>>(p, value, n);
  return lsh_check_launch("fill_i32_kernel");
}

__global__ void sample_state_setup_kernel(SampleState* st, int n, unsigned long long seed) {
  const int i = blockIdx.x * blockDim.x + threadIdx.x;
  if (i < n) st[i] = SampleState{seed, (unsigned)i, 0u};
}

int sample_state_setup(void* state, int n, unsigned long long seed, hipStream_t s) {
  if (!state || n <= 0 || (reinterpret_cast<uintptr_t>(state) & 15u) != 0)
    return lsh_fail(LSH_ERR_INVALID, "rng_setup: needs a 16-byte aligned state array");
  sample_state_setup_kernel<<<(n + 255) / 256, 256, 0, s>>>(static_cast<SampleState*>(state), n,
                                                            seed);
  return lsh_check_launch("sample_state_setup_kernel");
}

}  // namespace lsh

using namespace lsh;

extern "C" {

const char* lsh_last_error(void) { return g_last_error.c_str(); }
const char* lsh_version(void) { return "lightseq_hip 0.1 (gfx950)"; }

}  // extern "C"
