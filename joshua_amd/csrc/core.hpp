// What every translation unit of libjoshua_hip.so shares on the host: the error text, device selection, weight
// objects, and the scratch memory a call's launches hand to each other.
#pragma once
#include <hip/hip_runtime.h>

#include <algorithm>
#include <cmath>
#include <cstdio>
#include <cstdlib>
#include <cstring>
#include <map>
#include <memory>
#include <mutex>
#include <set>
#include <string>
#include <tuple>
#include <vector>

#include "../../include/joshua_hip.h"

struct jq_weight {
    uint32_t type;
    // nbytes: the elements alone.  Rows of the dense types (BF16, F32) start row_bytes apart, a whole number of
    // 64 elements, with zeros behind the k-th.
    size_t n, k, nbytes, row_bytes;
    uint8_t *dev;
    bool owns;
};

namespace jqh {

int fail(const char *fmt, ...) __attribute__((format(printf, 1, 2)));
void note_kernel(const char *name);  // what jq_last_kernel reports

#define HIP_TRY(expr)                                                                      \
    do {                                                                                   \
        hipError_t e_ = (expr);                                                            \
        if (e_ != hipSuccess) return fail("%s: %s", #expr, hipGetErrorString(e_));         \
    } while (0)

struct Geometry {
    size_t elems, bytes;
};
bool geometry(uint32_t t, Geometry *g);  // block formats only
const char *type_name(uint32_t t);
// Bytes of an element of the types held as plain rows (BF16: 2, F32: 4), else 0.
size_t dense_elem_bytes(uint32_t t);
constexpr size_t DENSE_PAD = 64;  // elements a dense row is padded to
inline size_t dense_stride(size_t k) { return (k + DENSE_PAD - 1) / DENSE_PAD * DENSE_PAD; }

int ensure_init();
int current_device_index();
int noalloc_scratch_on(int device, uint8_t **out);
std::mutex &noalloc_scratch_mutex(int device);
int release_stream_scratch(hipStream_t s);

struct FixedScratch {
    uint8_t *ptr = nullptr;
    size_t bytes = 0;
    std::mutex *mu = nullptr;
};
extern thread_local const FixedScratch *tl_fixed_scratch;

struct FixedScratchScope {
    explicit FixedScratchScope(const FixedScratch *f) { tl_fixed_scratch = f; }
    ~FixedScratchScope() { tl_fixed_scratch = nullptr; }
};

// Device memory for what one call's launches hand to each other (prepared activation operands, partial
// sums of a product split over k), on stream s.  Requests up to SCRATCH_KEEP bytes are served from one
// allocation per (device, stream), made at first use and kept until the process ends: the launches of a
// stream run in order, so consecutive calls can share it, and a call pays no allocator round trip
// (hipMallocAsync with hipFreeAsync takes some 18 us of host time a call, more than the kernels of a
// small matmul take on the device).  A call that needs more than the stream's buffer holds gets a new,
// larger one; the old one is retired, not freed, because a HIP graph captured earlier on the stream
// still names it (sizes at least double, so a stream retires at most a handful of buffers).  The holder
// keeps that allocation's lock until it goes out of scope, after the call's last launch is enqueued, so
// host threads that share a stream enqueue their calls one after the other.  Larger requests are
// stream-ordered allocations, freed behind the call's launches.  First use and growth allocate: neither
// is possible while the stream is being captured, so a caller warms a stream up with its largest call
// before capturing it.
//
// jq_matmul_t_noalloc serves the same requests from a fixed array in device memory instead (below): it
// installs the array for the calling thread with FixedScratchScope, and get() then hands out that
// array, or fails when the request exceeds it, and never reaches an allocator.
constexpr size_t SCRATCH_KEEP = 64u << 20;
class CallScratch {
    std::unique_lock<std::mutex> lock_;
    hipStream_t stream_ = nullptr;
    uint8_t *transient_ = nullptr;
    int kind_ = 0;

public:
    CallScratch() = default;
    explicit CallScratch(int kind) : kind_(kind) {}
    CallScratch(const CallScratch &) = delete;
    CallScratch &operator=(const CallScratch &) = delete;
    ~CallScratch();
    // 0 on success; on failure the message is set
    int get(size_t bytes, hipStream_t s, uint8_t **out);
};

// Frees a device allocation when it goes out of scope.
struct DevBuf {
    void *p = nullptr;
    DevBuf() = default;
    DevBuf(const DevBuf &) = delete;
    DevBuf &operator=(const DevBuf &) = delete;
    ~DevBuf() {
        if (p) (void)hipFree(p);
    }
    hipError_t alloc(size_t bytes) { return hipMalloc(&p, bytes ? bytes : 1); }
};

inline unsigned grid_for(size_t total) { return (unsigned)std::min<size_t>((total + 255) / 256, 8192); }

}  // namespace jqh

using namespace jqh;
