// Error text, device selection, the scratch memory behind calls, and weight objects (declared in core.hpp and
// include/joshua_hip.h).
#include <cstdarg>

#include "core.hpp"

namespace jqh {

thread_local char g_err[512] = "";
// Name of the kernel the calling thread's last matmul dispatch chose (jq_last_kernel).
thread_local const char *g_last_kernel = "";
void note_kernel(const char *name) { g_last_kernel = name; }

int fail(const char *fmt, ...) {
    va_list ap;
    va_start(ap, fmt);
    vsnprintf(g_err, sizeof g_err, fmt, ap);
    va_end(ap);
    return 1;
}

bool geometry(uint32_t t, Geometry *g) {
    switch (t) {  // reference: src/gguf_ext.rs:483-512
    case JQ_TYPE_Q8_0: *g = {32, 34}; return true;
    case JQ_TYPE_Q2_K: *g = {256, 84}; return true;
    case JQ_TYPE_Q4_K: *g = {256, 144}; return true;
    case JQ_TYPE_Q6_K: *g = {256, 210}; return true;
    case JQ_TYPE_IQ2_XXS: *g = {256, 66}; return true;
    case JQ_TYPE_MXFP4: *g = {32, 17}; return true;
    case JQ_TYPE_Q4_0: *g = {32, 18}; return true;
    case JQ_TYPE_Q4_1: *g = {32, 20}; return true;
    case JQ_TYPE_Q5_0: *g = {32, 22}; return true;
    case JQ_TYPE_Q5_1: *g = {32, 24}; return true;
    case JQ_TYPE_Q3_K: *g = {256, 110}; return true;
    case JQ_TYPE_Q5_K: *g = {256, 176}; return true;
    default: return false;
    }
}

size_t dense_elem_bytes(uint32_t t) { return t == JQ_TYPE_BF16 ? 2 : t == JQ_TYPE_F32 ? 4 : 0; }

const char *type_name(uint32_t t) {
    switch (t) {
    case JQ_TYPE_F32: return "f32";
    case JQ_TYPE_BF16: return "bf16";
    case JQ_TYPE_Q8_0: return "quantized";
    case JQ_TYPE_Q2_K: return "quantized";
    case JQ_TYPE_Q4_K: return "quantized";
    case JQ_TYPE_Q6_K: return "quantized";
    case JQ_TYPE_Q4_0: case JQ_TYPE_Q4_1: case JQ_TYPE_Q5_0: case JQ_TYPE_Q5_1: case JQ_TYPE_Q3_K: case JQ_TYPE_Q5_K:
        return "quantized";
    case JQ_TYPE_IQ2_XXS: return "iq2_xxs";
    case JQ_TYPE_MXFP4: return "mxfp4";
    default: return "unknown";
    }
}

std::once_flag g_init_once;
int g_init_rc = 0;
int g_device = 0;
int current_device_index() { return g_device; }

}  // namespace jqh

// Scratch memory of jq_matmul_t_noalloc: a fixed array in every device's memory, held from the moment the
// library is loaded on that device until the process ends.  Host code never uses the array's name as an
// address (on the host it is a stand-in, not device memory): noalloc_scratch_on() asks the runtime for the
// array's address on a device, once, with that device current, and every launch gets that pointer.
static __device__ __align__(256) uint8_t scratch[JQ_NOALLOC_SCRATCH_BYTES];

namespace jqh {

constexpr int MAX_DEVICES = 64;
uint8_t *g_scratch_ptr[MAX_DEVICES] = {};
std::mutex g_scratch_mu[MAX_DEVICES];  // one call at a time enqueues launches that use a device's array
std::mutex g_scratch_table_mu;

// The address of `scratch` on `device`, which must be the current device.
int noalloc_scratch_on(int device, uint8_t **out) {
    if (device < 0 || device >= MAX_DEVICES) return fail("device %d is beyond the %d this library keeps scratch for", device, MAX_DEVICES);
    std::lock_guard<std::mutex> g(g_scratch_table_mu);
    if (!g_scratch_ptr[device]) {
        void *p = nullptr;
        HIP_TRY(hipGetSymbolAddress(&p, HIP_SYMBOL(scratch)));
        if (!p) return fail("hipGetSymbolAddress returned no address for the scratch array on device %d", device);
        g_scratch_ptr[device] = (uint8_t *)p;
    }
    *out = g_scratch_ptr[device];
    return 0;
}

int do_init(int device) {
    int count = 0;
    HIP_TRY(hipGetDeviceCount(&count));
    if (device < 0 || device >= count) return fail("jq_init: device %d out of range (%d visible)", device, count);
    HIP_TRY(hipSetDevice(device));
    g_device = device;
    uint8_t *p = nullptr;
    return noalloc_scratch_on(device, &p);
}

int ensure_init() {
    std::call_once(g_init_once, [] { g_init_rc = do_init(0); });
    return g_init_rc;
}
std::mutex &noalloc_scratch_mutex(int device) { return g_scratch_mu[device]; }

struct StreamBuffer {
    std::mutex mu;
    uint8_t *ptr = nullptr;
    size_t bytes = 0;
    std::vector<uint8_t *> retired;
};

std::mutex g_stream_table_mu;
// keyed by (device, stream, kind): kind 0 is what a product's launches hand to each other, kind 1 the f32 copies of
// jq_matmul_t_f16's operands around such a product (which takes buffer 0 itself)
std::map<std::tuple<int, hipStream_t, int>, std::unique_ptr<StreamBuffer>> g_stream_table;

// jq_stream_release: waits for the stream, then frees its buffer and the retired ones.
int release_stream_scratch(hipStream_t s) {
    int dev = 0;
    HIP_TRY(hipGetDevice(&dev));
    std::vector<std::unique_ptr<StreamBuffer>> bufs;
    {
        std::lock_guard<std::mutex> g(g_stream_table_mu);
        for (int kind = 0; kind < 2; kind++) {
            auto it = g_stream_table.find({dev, s, kind});
            if (it == g_stream_table.end()) continue;
            bufs.push_back(std::move(it->second));
            g_stream_table.erase(it);
        }
    }
    if (bufs.empty()) return 0;
    for (auto &b : bufs) { std::lock_guard<std::mutex> wait_for_the_last_holder(b->mu); }
    HIP_TRY(hipStreamSynchronize(s));
    for (auto &b : bufs) {
        if (b->ptr) (void)hipFree(b->ptr);
        for (uint8_t *p : b->retired) (void)hipFree(p);
    }
    return 0;
}

thread_local const FixedScratch *tl_fixed_scratch = nullptr;

CallScratch::~CallScratch() {
    if (transient_) (void)hipFreeAsync(transient_, stream_);
}

int CallScratch::get(size_t bytes, hipStream_t s, uint8_t **out) {
    stream_ = s;
    if (const FixedScratch *f = kind_ == 0 ? tl_fixed_scratch : nullptr) {
        if (bytes > f->bytes)
            return fail("this product needs %zu bytes of scratch memory; the entry point that allocates nothing "
                        "holds %zu", bytes, f->bytes);
        lock_ = std::unique_lock<std::mutex>(*f->mu);
        *out = f->ptr;
        return 0;
    }
    if (bytes > SCRATCH_KEEP) {
        HIP_TRY(hipMallocAsync((void **)&transient_, bytes, s));
        *out = transient_;
        return 0;
    }
    int dev = 0;
    HIP_TRY(hipGetDevice(&dev));
    StreamBuffer *b;
    {
        std::lock_guard<std::mutex> g(g_stream_table_mu);
        auto &slot = g_stream_table[{dev, s, kind_}];
        if (!slot) slot.reset(new StreamBuffer);
        b = slot.get();
    }
    lock_ = std::unique_lock<std::mutex>(b->mu);
    if (b->bytes < bytes) {
        const size_t want = std::min(SCRATCH_KEEP, std::max<size_t>({(bytes + 0xFFFFF) & ~(size_t)0xFFFFF, 2 * b->bytes,
                                                                      (size_t)1 << 20}));
        uint8_t *fresh = nullptr;
        HIP_TRY(hipMalloc((void **)&fresh, want));
        if (b->ptr) b->retired.push_back(b->ptr);
        b->ptr = fresh, b->bytes = want;
    }
    *out = b->ptr;
    return 0;
}

}  // namespace jqh

extern "C" {

const char *jq_last_error(void) { return g_err; }
const char *jq_last_kernel(void) { return g_last_kernel; }

int jq_block_geometry(uint32_t ggml_type, size_t *elems, size_t *bytes) {
    Geometry g;
    if (!geometry(ggml_type, &g)) return fail("unsupported tensor type id %u", ggml_type);
    if (elems) *elems = g.elems;
    if (bytes) *bytes = g.bytes;
    return 0;
}

int jq_init(int device) {
    bool first = false;
    std::call_once(g_init_once, [&] {
        first = true;
        g_init_rc = do_init(device);
    });
    if (!first && g_init_rc == 0 && device != g_device)
        return fail("jq_init: already initialised on device %d", g_device);
    return g_init_rc;
}

static int upload_dense(uint32_t type, size_t eb, const void *rows, size_t nbytes, size_t n, size_t k, int src_is_device,
                        jq_weight **out) {
    if (nbytes != n * k * eb)
        return fail("%s tensor: %zu bytes for %zu x %zu elements (expected %zu)", type_name(type), nbytes, n, k, n * k * eb);
    if (nbytes && !rows) return fail("jq_upload: blocks is null");
    if (ensure_init()) return 1;
    const size_t pitch = dense_stride(k) * eb;
    uint8_t *dev = nullptr;
    HIP_TRY(hipMalloc((void **)&dev, n * pitch + 64));
    hipError_t e = hipMemset(dev, 0, n * pitch + 64);
    if (e == hipSuccess && nbytes)
        e = hipMemcpy2D(dev, pitch, rows, k * eb, k * eb, n, src_is_device ? hipMemcpyDeviceToDevice : hipMemcpyHostToDevice);
    if (e != hipSuccess) {
        (void)hipFree(dev);
        return fail("jq_upload: copy to device failed: %s", hipGetErrorString(e));
    }
    *out = new jq_weight{type, n, k, nbytes, pitch, dev, true};
    return 0;
}

int jq_upload(uint32_t ggml_type, const void *blocks, size_t nbytes, size_t n, size_t k, int src_is_device,
              jq_weight **out) {
    if (!out) return fail("jq_upload: out is null");
    *out = nullptr;
    if (const size_t eb = dense_elem_bytes(ggml_type)) return upload_dense(ggml_type, eb, blocks, nbytes, n, k, src_is_device, out);
    Geometry g;
    if (!geometry(ggml_type, &g)) return fail("unsupported tensor type id %u", ggml_type);
    if (k % g.elems != 0)
        return fail("%s tensor: k=%zu is not a multiple of the block size %zu", type_name(ggml_type), k, g.elems);
    size_t want = n * (k / g.elems) * g.bytes;
    if (nbytes != want)
        return fail("%s tensor: %zu bytes for %zu x %zu elements (expected %zu)", type_name(ggml_type), nbytes, n, k,
                    want);
    if (nbytes && !blocks) return fail("jq_upload: blocks is null");
    if (ensure_init()) return 1;
    uint8_t *dev = nullptr;
    // Kernels read a row in 16-byte pieces that may start before the unit they
    // need; 64 spare bytes keep every such read inside the allocation.
    HIP_TRY(hipMalloc((void **)&dev, nbytes + 64));
    hipError_t e = hipMemcpy(dev, blocks, nbytes, src_is_device ? hipMemcpyDeviceToDevice : hipMemcpyHostToDevice);
    if (e == hipSuccess) e = hipMemset(dev + nbytes, 0, 64);
    if (e != hipSuccess) {
        (void)hipFree(dev);
        return fail("jq_upload: copy to device failed: %s", hipGetErrorString(e));
    }
    *out = new jq_weight{ggml_type, n, k, nbytes, (k / g.elems) * g.bytes, dev, true};
    return 0;
}

int jq_view(const jq_weight *parent, size_t byte_offset, size_t n, size_t k, jq_weight **out) {
    if (!out) return fail("jq_view: out is null");
    *out = nullptr;
    if (!parent) return fail("jq_view: parent is null");
    if (const size_t eb = dense_elem_bytes(parent->type)) {  // whole rows; the offset counts elements, not padding
        if (k != parent->k || byte_offset % (k * eb) != 0)
            return fail("jq_view: a view of a %s tensor is a range of its rows", type_name(parent->type));
        const size_t row = byte_offset / (k * eb);
        if (row > parent->n || n > parent->n - row)
            return fail("jq_view: range %zu+%zu exceeds the parent's %zu bytes", byte_offset, n * k * eb, parent->nbytes);
        *out = new jq_weight{parent->type, n, k, n * k * eb, parent->row_bytes, parent->dev + row * parent->row_bytes, false};
        return 0;
    }
    Geometry g;
    geometry(parent->type, &g);
    if (k % g.elems != 0)
        return fail("%s tensor: k=%zu is not a multiple of the block size %zu", type_name(parent->type), k, g.elems);
    size_t need = n * (k / g.elems) * g.bytes;
    // reference: src/mmap_tensor.rs:105-110 (range must lie inside the mapping)
    if (byte_offset > parent->nbytes || need > parent->nbytes - byte_offset)
        return fail("jq_view: range %zu+%zu exceeds the parent's %zu bytes", byte_offset, need, parent->nbytes);
    if (byte_offset % g.bytes != 0) return fail("jq_view: offset %zu is not a whole number of blocks", byte_offset);
    *out = new jq_weight{parent->type, n, k, need, (k / g.elems) * g.bytes, parent->dev + byte_offset, false};
    return 0;
}

void jq_free(jq_weight *w) {
    if (!w) return;
    if (w->owns && w->dev) (void)hipFree(w->dev);
    delete w;
}

uint32_t jq_dtype(const jq_weight *w) { return w ? w->type : 0; }

size_t jq_rows(const jq_weight *w) { return w ? w->n : 0; }
size_t jq_cols(const jq_weight *w) { return w ? w->k : 0; }
size_t jq_storage_size_in_bytes(const jq_weight *w) { return w ? w->nbytes : 0; }
const void *jq_device_ptr(const jq_weight *w) { return w ? w->dev : nullptr; }

int jq_stream_release(void *stream) {
    if (ensure_init()) return 1;
    return release_stream_scratch((hipStream_t)stream);
}

int jq_stream_synchronize(void *stream) {
    HIP_TRY(hipStreamSynchronize((hipStream_t)stream));
    return 0;
}

}  // extern "C"
