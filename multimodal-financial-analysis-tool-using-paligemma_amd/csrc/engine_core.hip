// engine_core.hip -- the family-independent part of libpgmi's C ABI (include/pgmi.h): errors, the weight
// slab and its loaders, prepare / cache-size dispatch, token picking (argmax, top-p, stop tokens) and the
// replicas' load-time broadcast.
#include <dlfcn.h>

#include <rccl/rccl.h>  // types only: librccl is dlopen'ed on first use

#include "engine.h"
#include "safetensors_hdr.h"

static thread_local std::string g_err;

int pgmi_fail(int code, const std::string& msg) {
    g_err = msg;
    return code;
}

namespace {

__global__ void k_convert(const void* src, int dtype, long n, uint16_t* dst) {
    for (long i = blockIdx.x * (long)blockDim.x + threadIdx.x; i < n; i += (long)gridDim.x * blockDim.x) {
        if (dtype == PGMI_DTYPE_F32) dst[i] = f2bf(reinterpret_cast<const float*>(src)[i]);
        else dst[i] = f2bf((float)reinterpret_cast<const _Float16*>(src)[i]);
    }
}

}  // namespace

// RCCL is loaded on first use (dlopen), so a single-GPU process -- and the CPU tests that only load
// the library -- need no librccl; the four entry points it uses are resolved once.
namespace {
struct Rccl {
    void* h = nullptr;
    std::string why;  // dlerror() of the failed load
    ncclResult_t (*get_unique_id)(ncclUniqueId*) = nullptr;
    ncclResult_t (*comm_init_rank)(ncclComm_t*, int, ncclUniqueId, int) = nullptr;
    ncclResult_t (*comm_destroy)(ncclComm_t) = nullptr;
    ncclResult_t (*broadcast)(const void*, void*, size_t, ncclDataType_t, int, ncclComm_t, hipStream_t) = nullptr;
    const char* (*error_string)(ncclResult_t) = nullptr;
};

// thread-safe one-time load (a function-local static is initialised exactly once)
Rccl& rccl() {
    static Rccl r = [] {
        Rccl t;
        for (const char* n : {"librccl.so.1", "librccl.so", "/opt/rocm/lib/librccl.so.1"}) {
            if ((t.h = dlopen(n, RTLD_NOW | RTLD_LOCAL))) break;
            const char* e = dlerror();
            if (e) t.why = e;
        }
        if (t.h) {
            t.get_unique_id = reinterpret_cast<decltype(t.get_unique_id)>(dlsym(t.h, "ncclGetUniqueId"));
            t.comm_init_rank = reinterpret_cast<decltype(t.comm_init_rank)>(dlsym(t.h, "ncclCommInitRank"));
            t.comm_destroy = reinterpret_cast<decltype(t.comm_destroy)>(dlsym(t.h, "ncclCommDestroy"));
            t.broadcast = reinterpret_cast<decltype(t.broadcast)>(dlsym(t.h, "ncclBroadcast"));
            t.error_string = reinterpret_cast<decltype(t.error_string)>(dlsym(t.h, "ncclGetErrorString"));
        }
        return t;
    }();
    return r;
}
}  // namespace

extern "C" {

const char* pgmi_last_error(void) { return g_err.c_str(); }
const char* pgmi_version(void) { return "pgmi 0.1.0 (gfx950)"; }

int pgmi_destroy(pgmi_ctx* x) {
    if (x)
        for (auto& e : x->probe_ev) (void)hipEventDestroy(e);
    if (!x) return 0;
    clear_dgraphs(x);
    clear_pgraphs(x);
    if (x->release) x->release(x);
    for (void* p : x->allocs) (void)hipFree(p);
    if (x->cap_stream) (void)hipStreamDestroy(x->cap_stream);
    delete x;
    return 0;
}

int64_t pgmi_weights_bytes(const pgmi_ctx* x) { return x ? x->slab_bytes : -1; }
int pgmi_weight_count(const pgmi_ctx* x) { return x ? (int)x->slots.size() : -1; }

int pgmi_weight_info(const pgmi_ctx* x, int idx, const char** name, int64_t* off, int64_t* shape4, int* ndim) {
    if (!x || idx < 0 || idx >= (int)x->slots.size()) return fail(PGMI_E_ARG, "weight index out of range");
    const Slot& s = x->slots[idx];
    if (name) *name = s.name.c_str();
    if (off) *off = s.off;
    if (shape4) for (int i = 0; i < 4; ++i) shape4[i] = s.shape[i];
    if (ndim) *ndim = s.ndim;
    return 0;
}

int pgmi_bind_weights(pgmi_ctx* x, void* slab) {
    if (!x || !slab) return fail(PGMI_E_ARG, "null argument");
    if (reinterpret_cast<uintptr_t>(slab) % 256 != 0) return fail(PGMI_E_ARG, "weight slab must be 256-byte aligned");
    x->slab = reinterpret_cast<uint8_t*>(slab);
    clear_dgraphs(x);
    clear_pgraphs(x);
    return 0;
}

int pgmi_load_weight(pgmi_ctx* x, const char* name, const void* src, int dtype, int on_device, void* stream) {
    if (!x || !name || !src) return fail(PGMI_E_ARG, "null argument");
    if (!x->slab) return fail(PGMI_E_STATE, "weights are not bound");
    auto it = x->index.find(name);
    if (it == x->index.end()) return fail(PGMI_E_ARG, std::string("unknown weight ") + name);
    const Slot& s = x->slots[it->second];
    uint16_t* dst = reinterpret_cast<uint16_t*>(x->slab + s.off);
    hipStream_t st = (hipStream_t)stream;
    HIPCHK(hipSetDevice(x->device));
    if (dtype == PGMI_DTYPE_BF16) {
        HIPCHK(hipMemcpyAsync(dst, src, s.numel * 2, on_device ? hipMemcpyDeviceToDevice : hipMemcpyHostToDevice, st));
    } else if (dtype == PGMI_DTYPE_F32 || dtype == PGMI_DTYPE_F16) {
        if (on_device) {
            hipLaunchKernelGGL(k_convert, dim3(1024), dim3(256), 0, st, src, dtype, (long)s.numel, dst);
            LAUNCHCHK();
        } else {
            std::vector<uint16_t> tmp(s.numel);
            for (int64_t i = 0; i < s.numel; ++i) {
                float f = dtype == PGMI_DTYPE_F32 ? reinterpret_cast<const float*>(src)[i]
                                                 : (float)reinterpret_cast<const _Float16*>(src)[i];
                tmp[i] = host_f2bf(f);
            }
            HIPCHK(hipMemcpyAsync(dst, tmp.data(), s.numel * 2, hipMemcpyHostToDevice, st));
            HIPCHK(hipStreamSynchronize(st));
        }
    } else {
        return fail(PGMI_E_ARG, "unsupported dtype");
    }
    return 0;
}

int pgmi_safetensors_count(const char* path, int* n) {
    if (!path || !n) return fail(PGMI_E_ARG, "null argument");
    StFile f;
    if (!st_open(path, f)) return fail(PGMI_E_ARG, f.error);
    *n = (int)f.entries.size();
    return 0;
}

int pgmi_safetensors_entry(const char* path, int i, char* name, int name_cap, int* dtype, int64_t* shape4, int* ndim,
                           int64_t* begin, int64_t* end) {
    if (!path || !name || name_cap < 1 || !dtype || !shape4 || !ndim || !begin || !end)
        return fail(PGMI_E_ARG, "null argument");
    StFile f;
    if (!st_open(path, f)) return fail(PGMI_E_ARG, f.error);
    if (i < 0 || i >= (int)f.entries.size()) return fail(PGMI_E_ARG, "entry index out of range");
    const StEntry& e = f.entries[i];
    std::snprintf(name, (size_t)name_cap, "%s", e.name.c_str());
    *dtype = e.dtype == "BF16" ? PGMI_DTYPE_BF16 : e.dtype == "F16" ? PGMI_DTYPE_F16 : e.dtype == "F32" ? PGMI_DTYPE_F32 : -1;
    *ndim = (int)e.shape.size();
    for (int d = 0; d < 4; ++d) shape4[d] = d < *ndim ? e.shape[d] : 0;
    *begin = e.begin;
    *end = e.end;
    return 0;
}

// utils.py:19-44 (safe_open shard loop + load_state_dict(strict=False)) for one shard: tensors
// named like slab weights are shape-checked, converted to bf16 and written into the slab; BF16
// bytes go host -> slab directly from the mapped file, F32/F16 through the split-K scratch in
// chunks and a device-side RNE conversion.  Synchronises the stream before unmapping.
int pgmi_load_safetensors(pgmi_ctx* x, const char* path, int* n_loaded, int* n_skipped, void* stream) {
    if (!x || !path) return fail(PGMI_E_ARG, "null argument");
    if (!x->slab) return fail(PGMI_E_STATE, "weights are not bound");
    HIPCHK(hipSetDevice(x->device));
    StFile f;
    if (!st_open(path, f)) return fail(PGMI_E_ARG, f.error);
    hipStream_t st = (hipStream_t)stream;
    // scratch for conversions: the context's workspace if prepared, else a temporary buffer
    void* tmp = nullptr;
    size_t tmp_bytes = 0;
    uint8_t* scratch = reinterpret_cast<uint8_t*>(x->ws);
    size_t scratch_bytes = x->ws ? x->ws_bytes : 0;
    int loaded = 0, skipped = 0;
    int rc = 0;
    for (const StEntry& e : f.entries) {
        auto it = x->index.find(e.name);
        if (it == x->index.end()) {
            ++skipped;
            continue;
        }
        const Slot& sl = x->slots[it->second];
        bool same = (int)e.shape.size() == sl.ndim;
        for (int d = 0; same && d < sl.ndim; ++d) same = e.shape[d] == sl.shape[d];
        if (!same) {
            rc = fail(PGMI_E_ARG, "shape mismatch for " + e.name);
            break;
        }
        const int eb = st_elem_bytes(e.dtype);
        if (eb == 0) {
            rc = fail(PGMI_E_ARG, "unsupported dtype " + e.dtype + " for " + e.name);
            break;
        }
        if (e.end - e.begin != sl.numel * eb) {
            rc = fail(PGMI_E_ARG, "byte size mismatch for " + e.name);
            break;
        }
        const uint8_t* src = f.map + f.data0 + e.begin;
        uint16_t* dst = reinterpret_cast<uint16_t*>(x->slab + sl.off);
        if (e.dtype == "BF16") {
            if (hipMemcpyAsync(dst, src, (size_t)sl.numel * 2, hipMemcpyHostToDevice, st) != hipSuccess) {
                rc = fail(PGMI_E_HIP, "upload of " + e.name);
                break;
            }
        } else {
            const int dt = e.dtype == "F32" ? PGMI_DTYPE_F32 : PGMI_DTYPE_F16;
            if (scratch_bytes < ((size_t)8 << 20)) {
                if (!tmp) {
                    tmp_bytes = (size_t)64 << 20;
                    if (hipMalloc(&tmp, tmp_bytes) != hipSuccess) {
                        rc = fail(PGMI_E_NOMEM, "conversion scratch");
                        break;
                    }
                }
                scratch = reinterpret_cast<uint8_t*>(tmp);
                scratch_bytes = tmp_bytes;
            }
            const int64_t per = (int64_t)(scratch_bytes / (size_t)eb);
            for (int64_t i0 = 0; i0 < sl.numel && rc == 0; i0 += per) {
                const int64_t n = std::min<int64_t>(per, sl.numel - i0);
                if (hipMemcpyAsync(scratch, src + i0 * eb, (size_t)n * eb, hipMemcpyHostToDevice, st) != hipSuccess) {
                    rc = fail(PGMI_E_HIP, "upload of " + e.name);
                    break;
                }
                hipLaunchKernelGGL(k_convert, dim3(1024), dim3(256), 0, st, scratch, dt, (long)n, dst + i0);
            }
            if (rc) break;
        }
        ++loaded;
    }
    const hipError_t se = hipStreamSynchronize(st);  // the mapped bytes must outlive the copies
    if (tmp) (void)hipFree(tmp);
    if (rc) return rc;
    if (se != hipSuccess) return fail(PGMI_E_HIP, std::string("safetensors upload: ") + hipGetErrorString(se));
    x->prepared = false;  // derived tensors (padded patch matrix, ...) are rebuilt by pgmi_prepare
    if (n_loaded) *n_loaded = loaded;
    if (n_skipped) *n_skipped = skipped;
    return 0;
}

uint64_t pgmi_synthetic_key(const char* name, uint64_t seed) { return splitmix64_h(seed ^ fnv1a(name)); }

int pgmi_fill_synthetic(pgmi_ctx* x, const char* name, uint64_t key, float scale, float offset, void* stream) {
    if (!x || !name) return fail(PGMI_E_ARG, "null argument");
    if (!x->slab) return fail(PGMI_E_STATE, "weights are not bound");
    auto it = x->index.find(name);
    if (it == x->index.end()) return fail(PGMI_E_ARG, std::string("unknown weight ") + name);
    const Slot& s = x->slots[it->second];
    HIPCHK(hipSetDevice(x->device));
    fill_synthetic((hipStream_t)stream, reinterpret_cast<uint16_t*>(x->slab + s.off), (long)s.numel, key, scale, offset);
    LAUNCHCHK();
    return 0;
}

int pgmi_prepare(pgmi_ctx* x) {
    if (!x) return fail(PGMI_E_ARG, "null argument");
    if (!x->slab) return fail(PGMI_E_STATE, "weights are not bound");
    HIPCHK(hipSetDevice(x->device));
    return x->prepare(x);
}

int64_t pgmi_kv_bytes(const pgmi_ctx* x, int batch, int max_tokens) {
    return x ? x->kv_bytes(x, batch, max_tokens) : -1;
}

// ---------------------------------------------------------------- replicas: load-time broadcast
#define RCCL_READY()                                                                       \
    do {                                                                                   \
        const Rccl& r_ = rccl();                                                           \
        if (!r_.get_unique_id || !r_.comm_init_rank || !r_.comm_destroy || !r_.broadcast || !r_.error_string) \
            return fail(PGMI_E_STATE, std::string("librccl could not be loaded (dlopen librccl.so.1): ") + \
                        (r_.h ? "missing nccl* symbols" : r_.why));                        \
    } while (0)

#define NCCLCHK(expr)                                                                      \
    do {                                                                                   \
        ncclResult_t r_ = (expr);                                                          \
        if (r_ != ncclSuccess) return fail(PGMI_E_HIP, std::string(#expr) + ": " + rccl().error_string(r_)); \
    } while (0)

int pgmi_comm_unique_id(void* id_out) {
    if (!id_out) return fail(PGMI_E_ARG, "null argument");
    RCCL_READY();
    static_assert(sizeof(ncclUniqueId) == PGMI_COMM_ID_BYTES, "ncclUniqueId size");
    ncclUniqueId id;
    NCCLCHK(rccl().get_unique_id(&id));
    std::memcpy(id_out, &id, sizeof(id));
    return 0;
}

int pgmi_comm_init(int device, int nranks, int rank, const void* id, void** comm_out) {
    if (!id || !comm_out) return fail(PGMI_E_ARG, "null argument");
    if (nranks < 1 || rank < 0 || rank >= nranks) return fail(PGMI_E_ARG, "bad rank / world size");
    RCCL_READY();
    // the communicator binds to the current device: switch for the init, then give the caller's
    // thread its own current device back (torch keeps its own notion of it)
    int prev = 0;
    HIPCHK(hipGetDevice(&prev));
    HIPCHK(hipSetDevice(device));
    ncclUniqueId uid;
    std::memcpy(&uid, id, sizeof(uid));
    ncclComm_t comm = nullptr;
    const ncclResult_t r = rccl().comm_init_rank(&comm, nranks, uid, rank);
    HIPCHK(hipSetDevice(prev));
    if (r != ncclSuccess) return fail(PGMI_E_HIP, std::string("ncclCommInitRank: ") + rccl().error_string(r));
    *comm_out = comm;
    return 0;
}

int pgmi_comm_destroy(void* comm) {
    if (!comm) return 0;
    RCCL_READY();
    NCCLCHK(rccl().comm_destroy(reinterpret_cast<ncclComm_t>(comm)));
    return 0;
}

int pgmi_broadcast_weights(pgmi_ctx* x, void* comm, int root, void* stream) {
    if (!x || !comm) return fail(PGMI_E_ARG, "null argument");
    if (!x->slab) return fail(PGMI_E_STATE, "weights are not bound (pgmi_bind_weights)");
    RCCL_READY();
    int prev = 0;
    HIPCHK(hipGetDevice(&prev));
    HIPCHK(hipSetDevice(x->device));
    // the whole slab in one in-place collective: rank `root`'s bytes land in every replica
    const ncclResult_t r = rccl().broadcast(x->slab, x->slab, (size_t)x->slab_bytes, ncclUint8, root,
                                            reinterpret_cast<ncclComm_t>(comm), (hipStream_t)stream);
    HIPCHK(hipSetDevice(prev));
    if (r != ncclSuccess) return fail(PGMI_E_HIP, std::string("ncclBroadcast: ") + rccl().error_string(r));
    x->prepared = false;  // derived tensors are rebuilt from the received weights by pgmi_prepare
    return 0;
}

int pgmi_argmax(pgmi_ctx* x, const float* logits, int rows, int V, int64_t* out, void* stream) {
    if (!x || !logits || !out) return fail(PGMI_E_ARG, "null argument");
    if (rows <= 0 || V <= 0) return fail(PGMI_E_ARG, "argmax: empty logits");
    if (!x->amax_v) return fail(PGMI_E_STATE, "argmax scratch missing");
    argmax_rows((hipStream_t)stream, logits, rows, V, x->amax_v, x->amax_i, out);
    LAUNCHCHK();
    return 0;
}

int pgmi_eos_update(pgmi_ctx* x, int64_t* next_ids, int32_t* finished, int B, int64_t eos_id, int64_t pad_id,
                    int32_t* n_alive, void* stream) {
    if (!x || !next_ids || !finished) return fail(PGMI_E_ARG, "null argument");
    if (B <= 0) return fail(PGMI_E_ARG, "eos_update: empty batch");
    eos_update((hipStream_t)stream, next_ids, finished, B, eos_id, pad_id, n_alive);
    LAUNCHCHK();
    return 0;
}
int pgmi_sample_top_p(pgmi_ctx* x, const float* logits, int rows, int V, float temperature, float top_p,
                      const float* u, int64_t* out, float* kept_mass, void* stream) {
    if (!x || !logits || !u || !out) return fail(PGMI_E_ARG, "null argument");
    if (rows <= 0 || V <= 0) return fail(PGMI_E_ARG, "sample_top_p: empty probabilities");
    if (!(top_p >= 0.f)) return fail(PGMI_E_ARG, "sample_top_p: top_p must be >= 0");
    if (!x->ws) return fail(PGMI_E_STATE, "workspace not allocated (pgmi_prepare)");
    const int per = (int)std::min<size_t>((size_t)rows, x->ws_bytes / sample_scratch_bytes(1, V));
    if (per < 1) return fail(PGMI_E_ARG, "sample_top_p: vocabulary exceeds the scratch");
    for (int r0 = 0; r0 < rows; r0 += per) {  // row batches that fit the scratch (stream-ordered)
        const int nr = std::min(per, rows - r0);
        sample_top_p((hipStream_t)stream, logits + (size_t)r0 * V, nr, V, temperature, top_p, u + r0, x->ws,
                     out + r0, kept_mass ? kept_mass + r0 : nullptr);
    }
    LAUNCHCHK();
    return 0;
}

}  // extern "C"
