// C ABI: context, device memory, events and weight upload, shared by every model family
// (see include/cera_hip.h for the contract of each).
#include <algorithm>
#include <cstdio>
#include <cstring>
#include <new>

#include "cera_hip_kernels.h"
#include "host_common.h"

// ---------------------------------------------------------------------------
// Fixed workspace of the allocation-free attention entry (cera_hip_attn_decode_dev_noalloc): the
// split-K partials of one decode-attention call.  The array's name is only a host-side handle;
// its device address is resolved once per device at context creation and that pointer is what
// kernels receive.  Every GPU holds its own copy until the process ends.
static __device__ __align__(256) unsigned char scratch[CERA_HIP_NOALLOC_WORKSPACE_BYTES];
static constexpr int MAX_DEVICES = 64;
static std::mutex g_scratch_mu;
static void* g_scratch_ptr[MAX_DEVICES] = {nullptr};

// with `device` current: the address of this device's copy of `scratch`
static hipError_t resolve_static_scratch(int device, void** out) {
    std::lock_guard<std::mutex> lk(g_scratch_mu);
    if (!g_scratch_ptr[device]) {
        void* p = nullptr;
        hipError_t e = hipGetSymbolAddress(&p, HIP_SYMBOL(scratch));
        if (e != hipSuccess) return e;
        g_scratch_ptr[device] = p;
    }
    *out = g_scratch_ptr[device];
    return hipSuccess;
}

static std::mutex g_err_mu;
static std::string g_err;

void cera_set_global_error(const std::string& s) {
    std::lock_guard<std::mutex> lk(g_err_mu);
    g_err = s;
}
cera_hip_status cera_fail(cera_hip_ctx* ctx, cera_hip_status st, const std::string& msg) {
    if (ctx) ctx->err = msg;
    cera_set_global_error(msg);
    return st;
}

bool cera_type_geometry(uint32_t t, uint32_t* e, uint32_t* b) {
    switch (t) {
        case CERA_HIP_F32: *e = 1; *b = 4; return true;
        case CERA_HIP_F16: case CERA_HIP_BF16: *e = 1; *b = 2; return true;
        case CERA_HIP_Q4_0: *e = 32; *b = 18; return true;
        case CERA_HIP_Q4_1: *e = 32; *b = 20; return true;
        case CERA_HIP_Q8_0: *e = 32; *b = 34; return true;
        case CERA_HIP_Q4_K: *e = 256; *b = 144; return true;
        case CERA_HIP_Q5_K: *e = 256; *b = 176; return true;
        case CERA_HIP_Q6_K: *e = 256; *b = 210; return true;
        default: return false;
    }
}

cera_hip_status cera_scratch(cera_hip_ctx* ctx, int slot, uint64_t nbytes, void** out) {
    if (nbytes == 0) nbytes = 256;
    if (ctx->scratch_bytes[slot] < nbytes) {
        if (ctx->scratch[slot]) {
            HIP_TRY(ctx, hipStreamSynchronize(ctx->stream));
            HIP_TRY(ctx, hipFree(ctx->scratch[slot]));
            ctx->scratch[slot] = nullptr;
            ctx->scratch_bytes[slot] = 0;
        }
        uint64_t want = (nbytes + 4095) & ~uint64_t(4095);
        HIP_TRY(ctx, hipMalloc(&ctx->scratch[slot], want));
        ctx->scratch_bytes[slot] = want;
    }
    *out = ctx->scratch[slot];
    return CERA_HIP_OK;
}

hipFunction_t cera_module_fn(cera_hip_ctx* ctx, const std::string& name) {
    if (!ctx->module) return nullptr;
    auto it = ctx->module_fns.find(name);
    if (it != ctx->module_fns.end()) return it->second;
    hipFunction_t f = nullptr;
    if (hipModuleGetFunction(&f, ctx->module, name.c_str()) != hipSuccess) {
        f = nullptr;
        (void)hipGetLastError();   // "not found" is an answer, not a sticky error
    }
    ctx->module_fns.emplace(name, f);
    return f;
}

cera_hip_status cera_module_launch(cera_hip_ctx* ctx, hipFunction_t f, uint32_t grid, uint32_t block, void* args) {
    void* params[] = {args};
    HIP_TRY(ctx, hipModuleLaunchKernel(f, grid, 1, 1, block, 1, 1, 0, ctx->stream, params, nullptr));
    return CERA_HIP_OK;
}

cera_hip_status cera_check_tensor(cera_hip_ctx* ctx, const cera_hip_tensor* t, uint64_t* row_bytes) {
    if (!t || !t->data) return cera_fail(ctx, CERA_HIP_ERR_ARGUMENT, "tensor or tensor data is null");
    uint32_t e, b;
    if (!cera_type_geometry(t->ggml_type, &e, &b))
        return cera_fail(ctx, CERA_HIP_ERR_UNSUPPORTED_DTYPE,
                         "no hip kernel for ggml type " + std::to_string(t->ggml_type));
    if (t->m == 0 || t->k == 0 || t->k % e)
        return cera_fail(ctx, CERA_HIP_ERR_SHAPE, "k=" + std::to_string(t->k) + " is not a whole number of " +
                                                      std::to_string(e) + "-element blocks (or m/k is zero)");
    *row_bytes = t->k / e * b;
    if (t->nbytes != t->m * *row_bytes)
        return cera_fail(ctx, CERA_HIP_ERR_SHAPE, "tensor nbytes " + std::to_string(t->nbytes) + " != m*row_bytes " +
                                                      std::to_string(t->m * *row_bytes));
    if (t->m > 0xFFFFFFFFull || t->k > 0xFFFFFFFFull) return cera_fail(ctx, CERA_HIP_ERR_SHAPE, "dimension exceeds 2^32");
    return CERA_HIP_OK;
}

extern "C" {

cera_hip_status cera_hip_ctx_create(int device, const char* hsaco_path, cera_hip_ctx** out) {
    if (!out) return cera_fail(nullptr, CERA_HIP_ERR_ARGUMENT, "cera_hip_ctx_create: out is null");
    *out = nullptr;
    int n = 0;
    hipError_t e = hipGetDeviceCount(&n);
    if (e != hipSuccess || n == 0)
        return cera_fail(nullptr, CERA_HIP_ERR_DEVICE,
                         std::string("no HIP device available: ") + (e != hipSuccess ? hipGetErrorString(e) : "count is 0"));
    if (device < 0 || device >= n || device >= MAX_DEVICES) return cera_fail(nullptr, CERA_HIP_ERR_ARGUMENT, "device index out of range");
    cera_hip_ctx* ctx = new (std::nothrow) cera_hip_ctx();
    if (!ctx) return cera_fail(nullptr, CERA_HIP_ERR_OOM, "host allocation failed");
    ctx->device = device;
    hipDeviceProp_t prop;
    if ((e = hipSetDevice(device)) != hipSuccess || (e = hipGetDeviceProperties(&prop, device)) != hipSuccess ||
        (e = resolve_static_scratch(device, &ctx->static_scratch)) != hipSuccess ||
        (e = hipStreamCreate(&ctx->stream)) != hipSuccess) {
        delete ctx;
        return cera_fail(nullptr, CERA_HIP_ERR_DEVICE, std::string("device init: ") + hipGetErrorString(e));
    }
    if (std::strncmp(prop.gcnArchName, "gfx950", 6) != 0) {
        std::string arch = prop.gcnArchName;
        (void)hipStreamDestroy(ctx->stream);
        delete ctx;
        return cera_fail(nullptr, CERA_HIP_ERR_DEVICE, "kernels are built for gfx950 only; device is " + arch);
    }
    ctx->n_cu = static_cast<uint32_t>(prop.multiProcessorCount);
    if (hsaco_path) {
        if ((e = hipModuleLoad(&ctx->module, hsaco_path)) != hipSuccess) {
            (void)hipGetLastError();   // the failed load must not surface as a later call's error
            (void)hipStreamDestroy(ctx->stream);
            delete ctx;
            return cera_fail(nullptr, CERA_HIP_ERR_DEVICE, std::string("hipModuleLoad(") + hsaco_path + "): " + hipGetErrorString(e));
        }
        if (!cera_module_fn(ctx, "cera_k_quantize_q8_0")) {
            (void)hipModuleUnload(ctx->module);
            (void)hipStreamDestroy(ctx->stream);
            delete ctx;
            return cera_fail(nullptr, CERA_HIP_ERR_ARGUMENT, std::string(hsaco_path) + " is not this library's code object (no cera_k_quantize_q8_0)");
        }
    }
    *out = ctx;
    return CERA_HIP_OK;
}

void cera_hip_ctx_destroy(cera_hip_ctx* ctx) {
    if (!ctx) return;
    (void)hipSetDevice(ctx->device);
    (void)hipStreamSynchronize(ctx->stream);
    for (auto& p : ctx->scratch)
        if (p) (void)hipFree(p);
    if (ctx->attn_acc) (void)hipFree(ctx->attn_acc);
    if (ctx->attn_ml) (void)hipFree(ctx->attn_ml);
    for (int i = 0; i < 2; ++i) {
        if (ctx->pin[i]) (void)hipHostFree(ctx->pin[i]);
        if (ctx->pin_ev[i]) (void)hipEventDestroy(ctx->pin_ev[i]);
    }
    if (ctx->word_host) (void)hipHostFree(ctx->word_host);
    if (ctx->module) (void)hipModuleUnload(ctx->module);
    (void)hipStreamDestroy(ctx->stream);
    delete ctx;
}

const char* cera_hip_last_error(const cera_hip_ctx* ctx) {
    if (ctx) return ctx->err.c_str();
    static thread_local std::string copy;
    std::lock_guard<std::mutex> lk(g_err_mu);
    copy = g_err;
    return copy.c_str();
}

cera_hip_status cera_hip_sync(cera_hip_ctx* ctx) {
    if (!ctx) return CERA_HIP_ERR_ARGUMENT;
    HIP_TRY(ctx, hipStreamSynchronize(ctx->stream));
    return CERA_HIP_OK;
}

cera_hip_status cera_hip_ctx_set_decode_copies(cera_hip_ctx* ctx, int enabled) {
    if (!ctx) return CERA_HIP_ERR_ARGUMENT;
    std::lock_guard<std::recursive_mutex> lk(ctx->op_mu);
    ctx->decode_copies = enabled != 0;
    return CERA_HIP_OK;
}

cera_hip_status cera_hip_device_info(cera_hip_ctx* ctx, char* name256, uint32_t* n_cu, uint64_t* hbm) {
    if (!ctx) return CERA_HIP_ERR_ARGUMENT;
    hipDeviceProp_t prop;
    HIP_TRY(ctx, hipGetDeviceProperties(&prop, ctx->device));
    if (name256) {
        std::snprintf(name256, 256, "%s (%s)", prop.name, prop.gcnArchName);
    }
    if (n_cu) *n_cu = static_cast<uint32_t>(prop.multiProcessorCount);
    if (hbm) *hbm = prop.totalGlobalMem;
    return CERA_HIP_OK;
}

// ---- memory / events --------------------------------------------------------
cera_hip_status cera_hip_malloc(cera_hip_ctx* ctx, uint64_t nbytes, void** out) {
    if (!ctx || !out) return CERA_HIP_ERR_ARGUMENT;
    *out = nullptr;
    HIP_TRY(ctx, hipMalloc(out, nbytes ? nbytes : 256));
    return CERA_HIP_OK;
}
cera_hip_status cera_hip_free(cera_hip_ctx* ctx, void* dev) {
    if (!ctx) return CERA_HIP_ERR_ARGUMENT;
    if (!dev) return CERA_HIP_OK;
    HIP_TRY(ctx, hipStreamSynchronize(ctx->stream));
    HIP_TRY(ctx, hipFree(dev));
    return CERA_HIP_OK;
}
cera_hip_status cera_hip_upload(cera_hip_ctx* ctx, void* dst, const void* src, uint64_t n) {
    if (!ctx || (!dst && n) || (!src && n)) return CERA_HIP_ERR_ARGUMENT;
    if (n == 0) return CERA_HIP_OK;
    HIP_TRY(ctx, hipMemcpyAsync(dst, src, n, hipMemcpyHostToDevice, ctx->stream));
    HIP_TRY(ctx, hipStreamSynchronize(ctx->stream));
    return CERA_HIP_OK;
}
// Device -> pageable host memory.  The runtime's own route for a pageable destination moves
// copies of up to a few MB at about 2 GB/s (0.26 ms for one row of logits) and large ones at
// 17 GB/s (it pins the destination).  Staged through two pinned chunks, the DMA of chunk i+1
// running while the CPU copies chunk i out, the same copies take 0.06 ms and run at 25 GB/s;
// only beyond PIN_DIRECT bytes is the runtime's route taken.
static constexpr uint64_t PIN_CHUNK = 1u << 20, PIN_DIRECT = 256u << 20;
cera_hip_status cera_hip_download(cera_hip_ctx* ctx, void* dst, const void* src, uint64_t n) {
    if (!ctx || (!dst && n) || (!src && n)) return CERA_HIP_ERR_ARGUMENT;
    if (n == 0) return CERA_HIP_OK;
    if (n >= PIN_DIRECT) {
        HIP_TRY(ctx, hipMemcpyAsync(dst, src, n, hipMemcpyDeviceToHost, ctx->stream));
        HIP_TRY(ctx, hipStreamSynchronize(ctx->stream));
        return CERA_HIP_OK;
    }
    std::lock_guard<std::mutex> lk(ctx->pin_mu);
    for (int i = 0; i < 2; ++i) {
        if (!ctx->pin[i]) HIP_TRY(ctx, hipHostMalloc(&ctx->pin[i], PIN_CHUNK, hipHostMallocDefault));
        if (!ctx->pin_ev[i]) HIP_TRY(ctx, hipEventCreateWithFlags(&ctx->pin_ev[i], hipEventDisableTiming));
    }
    const uint64_t n_chunks = (n + PIN_CHUNK - 1) / PIN_CHUNK;
    for (uint64_t i = 0; i <= n_chunks; ++i) {
        if (i < n_chunks) {   // chunk i-2, the last user of this pinned buffer, was copied out one turn ago
            const uint64_t off = i * PIN_CHUNK, len = std::min(PIN_CHUNK, n - off);
            HIP_TRY(ctx, hipMemcpyAsync(ctx->pin[i & 1], static_cast<const char*>(src) + off, len, hipMemcpyDeviceToHost, ctx->stream));
            HIP_TRY(ctx, hipEventRecord(ctx->pin_ev[i & 1], ctx->stream));
        }
        if (i >= 1) {
            const uint64_t j = i - 1, off = j * PIN_CHUNK, len = std::min(PIN_CHUNK, n - off);
            HIP_TRY(ctx, hipEventSynchronize(ctx->pin_ev[j & 1]));
            std::memcpy(static_cast<char*>(dst) + off, ctx->pin[j & 1], len);
        }
    }
    return CERA_HIP_OK;
}
cera_hip_status cera_hip_copy_dev(cera_hip_ctx* ctx, void* dst, const void* src, uint64_t n) {
    if (!ctx || (!dst && n) || (!src && n)) return CERA_HIP_ERR_ARGUMENT;
    if (n == 0) return CERA_HIP_OK;
    HIP_TRY(ctx, hipMemcpyAsync(dst, src, n, hipMemcpyDeviceToDevice, ctx->stream));
    return CERA_HIP_OK;
}
// Plain streaming copy, 16 bytes per lane per step: a kernel of exactly known HBM traffic
// (n read + n written) against which hardware byte counters can be calibrated.
static __global__ void __launch_bounds__(256) copy_kernel(uint4* __restrict__ dst, const uint4* __restrict__ src, uint64_t n16) {
    for (uint64_t i = uint64_t(blockIdx.x) * blockDim.x + threadIdx.x; i < n16; i += uint64_t(gridDim.x) * blockDim.x)
        dst[i] = src[i];
}
cera_hip_status cera_hip_copy_kernel(cera_hip_ctx* ctx, void* dst, const void* src, uint64_t n) {
    if (!ctx || !dst || !src) return CERA_HIP_ERR_ARGUMENT;
    if (n == 0 || n % 16 || (reinterpret_cast<uintptr_t>(dst) | reinterpret_cast<uintptr_t>(src)) % 16)
        return cera_fail(ctx, CERA_HIP_ERR_SHAPE, "copy_kernel: size and pointers must be multiples of 16 bytes");
    uint64_t n16 = n / 16;
    uint32_t blocks = static_cast<uint32_t>(std::min<uint64_t>((n16 + 255) / 256, uint64_t(ctx->n_cu) * 16));
    hipLaunchKernelGGL(copy_kernel, dim3(blocks), dim3(256), 0, ctx->stream, static_cast<uint4*>(dst),
                       static_cast<const uint4*>(src), n16);
    HIP_TRY(ctx, hipGetLastError());
    return CERA_HIP_OK;
}
cera_hip_status cera_hip_event_create(cera_hip_ctx* ctx, cera_hip_event** out) {
    if (!ctx || !out) return CERA_HIP_ERR_ARGUMENT;
    cera_hip_event* e = new (std::nothrow) cera_hip_event();
    if (!e) return cera_fail(ctx, CERA_HIP_ERR_OOM, "host allocation failed");
    hipError_t r = hipEventCreate(&e->ev);
    if (r != hipSuccess) {
        delete e;
        return cera_fail(ctx, CERA_HIP_ERR_DEVICE, std::string("hipEventCreate: ") + hipGetErrorString(r));
    }
    *out = e;
    return CERA_HIP_OK;
}
void cera_hip_event_destroy(cera_hip_event* e) {
    if (!e) return;
    (void)hipEventDestroy(e->ev);
    delete e;
}
cera_hip_status cera_hip_event_record(cera_hip_ctx* ctx, cera_hip_event* e) {
    if (!ctx || !e) return CERA_HIP_ERR_ARGUMENT;
    HIP_TRY(ctx, hipEventRecord(e->ev, ctx->stream));
    return CERA_HIP_OK;
}
cera_hip_status cera_hip_event_elapsed_ms(cera_hip_ctx* ctx, cera_hip_event* a, cera_hip_event* b, float* ms) {
    if (!ctx || !a || !b || !ms) return CERA_HIP_ERR_ARGUMENT;
    HIP_TRY(ctx, hipEventSynchronize(b->ev));
    HIP_TRY(ctx, hipEventElapsedTime(ms, a->ev, b->ev));
    return CERA_HIP_OK;
}

// ---- weights ------------------------------------------------------------------

static cera_hip_status alloc_dtensor(cera_hip_ctx* ctx, uint32_t dtype, uint64_t m, uint64_t k, uint64_t row_bytes,
                                     cera_hip_dtensor** out) {
    cera_hip_dtensor* d = new (std::nothrow) cera_hip_dtensor();
    if (!d) return cera_fail(ctx, CERA_HIP_ERR_OOM, "host allocation failed");
    d->dtype = dtype; d->m = m; d->k = k; d->row_bytes = row_bytes; d->nbytes = m * row_bytes;
    // 64 bytes of slack: a dead lane may read up to one unit past its own data
    hipError_t e = hipMalloc(reinterpret_cast<void**>(&d->dev), d->nbytes + 64);
    if (e != hipSuccess) {
        delete d;
        return cera_fail(ctx, e == hipErrorOutOfMemory ? CERA_HIP_ERR_OOM : CERA_HIP_ERR_DEVICE,
                         std::string("hipMalloc(weights): ") + hipGetErrorString(e));
    }
    *out = d;
    return CERA_HIP_OK;
}

cera_hip_status cera_hip_tensor_upload(cera_hip_ctx* ctx, const cera_hip_tensor* t, cera_hip_dtensor** out) {
    if (!ctx || !out) return CERA_HIP_ERR_ARGUMENT;
    *out = nullptr;
    uint64_t rb;
    CERA_TRY(cera_check_tensor(ctx, t, &rb));
    cera_hip_dtensor* d;
    CERA_TRY(alloc_dtensor(ctx, t->ggml_type, t->m, t->k, rb, &d));
    hipError_t e = hipMemcpyAsync(d->dev, t->data, d->nbytes, hipMemcpyHostToDevice, ctx->stream);
    if (e == hipSuccess) e = hipStreamSynchronize(ctx->stream);
    if (e != hipSuccess) {
        (void)hipFree(d->dev);
        delete d;
        return cera_fail(ctx, CERA_HIP_ERR_DEVICE, std::string("weight upload: ") + hipGetErrorString(e));
    }
    *out = d;
    return CERA_HIP_OK;
}

cera_hip_status cera_hip_tensor_clone(cera_hip_ctx* ctx, const cera_hip_dtensor* src, cera_hip_dtensor** out) {
    if (!ctx || !src || !out) return CERA_HIP_ERR_ARGUMENT;
    *out = nullptr;
    cera_hip_dtensor* d;
    CERA_TRY(alloc_dtensor(ctx, src->dtype, src->m, src->k, src->row_bytes, &d));
    hipError_t e = hipMemcpyAsync(d->dev, src->dev, d->nbytes, hipMemcpyDeviceToDevice, ctx->stream);
    if (e == hipSuccess) e = hipStreamSynchronize(ctx->stream);
    if (e != hipSuccess) {
        (void)hipFree(d->dev);
        delete d;
        return cera_fail(ctx, CERA_HIP_ERR_DEVICE, std::string("weight clone: ") + hipGetErrorString(e));
    }
    *out = d;
    return CERA_HIP_OK;
}

void cera_hip_tensor_free(cera_hip_ctx* ctx, cera_hip_dtensor* d) {
    if (!d) return;
    if (ctx) (void)hipStreamSynchronize(ctx->stream);
    if (d->dev && d->owns) (void)hipFree(d->dev);
    if (d->dev_stream) (void)hipFree(d->dev_stream);
    delete d;
}
uint64_t cera_hip_tensor_nbytes(const cera_hip_dtensor* d) { return d ? d->nbytes : 0; }

}  // extern "C"

cera_hip_status cera_tensor_upload_concat(cera_hip_ctx* ctx, const cera_hip_tensor* const* parts, int n_parts,
                                          cera_hip_dtensor** fused, cera_hip_dtensor** views) {
    *fused = nullptr;
    uint64_t rb = 0, rows = 0;
    for (int i = 0; i < n_parts; ++i) {
        uint64_t r;
        CERA_TRY(cera_check_tensor(ctx, parts[i], &r));
        if (parts[i]->ggml_type != parts[0]->ggml_type || parts[i]->k != parts[0]->k)
            return cera_fail(ctx, CERA_HIP_ERR_SHAPE, "concat: parts differ in type or k");
        rb = r;
        rows += parts[i]->m;
    }
    cera_hip_dtensor* f;
    CERA_TRY(alloc_dtensor(ctx, parts[0]->ggml_type, rows, parts[0]->k, rb, &f));
    uint64_t off = 0;
    for (int i = 0; i < n_parts; ++i) {
        hipError_t e = hipMemcpyAsync(f->dev + off, parts[i]->data, parts[i]->nbytes, hipMemcpyHostToDevice, ctx->stream);
        if (e == hipSuccess) e = hipStreamSynchronize(ctx->stream);
        cera_hip_dtensor* v = e == hipSuccess ? new (std::nothrow) cera_hip_dtensor() : nullptr;
        if (!v) {
            for (int j = 0; j < i; ++j) { delete views[j]; views[j] = nullptr; }
            cera_hip_tensor_free(ctx, f);
            return cera_fail(ctx, e != hipSuccess ? CERA_HIP_ERR_DEVICE : CERA_HIP_ERR_OOM,
                             e != hipSuccess ? std::string("weight upload: ") + hipGetErrorString(e) : "host allocation failed");
        }
        v->dtype = f->dtype; v->m = parts[i]->m; v->k = f->k; v->row_bytes = rb; v->nbytes = parts[i]->nbytes;
        v->dev = f->dev + off; v->owns = false;
        views[i] = v;
        off += parts[i]->nbytes;
    }
    *fused = f;
    return CERA_HIP_OK;
}
