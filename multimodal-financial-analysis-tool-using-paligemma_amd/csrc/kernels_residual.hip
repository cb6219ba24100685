// kernels_residual.hip -- one residual stream: the embedding (with a table of token pairs), the scaled update from a
// finished sublayer (split-K slabs, a mixture's outputs), the RMS norm in front of the next one, a mixture's router behind
// that norm, and the causal input convolution added to what a mixer reads.  Stream, sums, norms, router and convolution
// are fp32.
#include <algorithm>

#include "act.h"
#include "decoder.h"
#include "route.h"

namespace pgmi {

namespace {

__device__ __forceinline__ void ldv(const float* p, float (&v)[4]) { ld4(p, v); }
__device__ __forceinline__ void ldv(const uint16_t* p, float (&v)[4]) { ld4(p, v); }
template <typename S>
__device__ __forceinline__ void ldv(const S* p, float (&v)[1]) { v[0] = ldf(p); }
template <typename S>
__device__ __forceinline__ void stv(S* p, const float (&v)[4]) { st4(p, v); }
template <typename S>
__device__ __forceinline__ void stv(S* p, const float (&v)[1]) { stf(p, v[0]); }

struct RouterArgs {
    const uint16_t* W;  // [n, and the gate's row][ldw]
    int ldw;
    RouteArgs r;
};

// One workgroup per row; PC pieces of V elements per thread, every load of a source issued before its first use.
// RT: the router of the row and its choice behind the norm, 16 waves; dynamic LDS: route_words(), then h [ldh].
// KT > 0: the input convolution's step with KT taps, its operands loaded ahead of the norm (0: any number, or none).
template <typename T, int V, int PC, bool RT, int KT>
__global__ void __launch_bounds__(1024) k_residual(ResidualArgs a, RouterArgs rt) {
    __shared__ float red[16];
    extern __shared__ __attribute__((aligned(16))) float rsm[];
    constexpr int RR = 4, RK = 4;  // router rows and 512-wide steps a wave has in flight
    const int rows_r = RT ? rt.r.n : 0;
    uint4 rw[RT ? RR : 1][RT ? RK : 1];
    auto rload = [&](int n0, int k0) {
        if constexpr (RT) {
#pragma unroll
            for (int q = 0; q < RR; ++q) {
                const uint16_t* p = rt.W + (long)min(n0 + 16 * q, rows_r - 1) * rt.ldw;
#pragma unroll
                for (int i = 0; i < RK; ++i) {
                    const int k = k0 + i * 512 + (threadIdx.x & 63) * 8;
                    rw[q][i] = ldg16_sel(p + k, k < a.ldh, p);
                }
            }
        }
    };
    const int tid = threadIdx.x, NT = blockDim.x, D = a.D;
    const int row = a.rows_idx ? a.rows_idx[blockIdx.x] : blockIdx.x;
    if (a.zero && blockIdx.x == 0)
        for (int i = tid; i < a.nzero; i += NT) a.zero[i] = 0;
    float* Xr = a.X + (long)row * D;
    float x[PC][V];
    int dd[PC];
    bool ok[PC];
#pragma unroll
    for (int i = 0; i < PC; ++i) {
        const int d = (i * NT + tid) * V;
        ok[i] = d < D;
        dd[i] = ok[i] ? d : 0;
    }
    int slot = 0, pos = 0;
    if (!a.seqs && a.slot) {
        slot = a.slot[row];
        pos = a.pos[row];
    }
    float* ring = a.taps > 0 ? a.ring + (long)slot * a.taps * D : nullptr;
    float wk[KT > 0 ? KT : 1][PC][V], back[KT > 1 ? KT - 1 : 1][PC][V];  // back[j]: the norm j + 1 positions ago
    if constexpr (KT > 0) {
#pragma unroll
        for (int i = 0; i < PC; ++i) {
#pragma unroll
            for (int v = 0; v < V; ++v)
#pragma unroll
                for (int j = 0; j < KT; ++j) wk[j][i][v] = bf2f(a.cw[(long)(dd[i] + v) * KT + j]);
#pragma unroll
            for (int j = 0; j < KT - 1; ++j) {
                const int p = pos - 1 - j;
                ldv(ring + (long)((p < 0 ? 0 : p) % KT) * D + dd[i], back[j][i]);
#pragma unroll
                for (int v = 0; v < V; ++v) back[j][i][v] = p < 0 ? 0.0f : back[j][i][v];
            }
        }
    }
    float gw[V];  // the gate's row of the router
#pragma unroll
    for (int v = 0; v < V; ++v) gw[v] = RT && rt.r.gate && ok[0] ? bf2f(rt.W[(long)rt.r.n * rt.ldw + dd[0] + v]) : 0.0f;
    if (a.ids) {
        long id = a.ids[row];
        id = id < 0 ? 0 : (id >= a.vocab ? a.vocab - 1 : id);
        const uint16_t* er = a.E + id * D;
#pragma unroll
        for (int i = 0; i < PC; ++i) {
            ldv(er + dd[i], x[i]);
#pragma unroll
            for (int v = 0; v < V; ++v) x[i][v] *= a.escale;
        }
        if (a.pairs) {
            bool here = false;  // the previous token is the row before this one
            if (a.seqs) {
                const SeqInfo q = a.seqs[a.row_seq[row]];
                slot = q.slot;
                pos = q.start + row - q.off;
                here = row > q.off;
            }
            int* hist = a.history + (long)slot * a.max_tokens + pos;
            long p = a.buckets;
            if (pos > 0) {
                long prev = here ? a.ids[row - 1] : hist[-1];
                prev = prev < 0 ? 0 : (prev >= a.vocab ? a.vocab - 1 : prev);
                p = (prev * a.mul_prev + id * a.mul_cur) % a.buckets;
            }
            if (tid == 0) *hist = (int)id;
            const uint16_t* pr = a.pairs + p * D;
#pragma unroll
            for (int i = 0; i < PC; ++i) {
                float q[V];
                ldv(pr + dd[i], q);
#pragma unroll
                for (int v = 0; v < V; ++v) x[i][v] += q[v];
            }
        }
    } else {
#pragma unroll
        for (int i = 0; i < PC; ++i) ldv(Xr + dd[i], x[i]);
    }
    if (a.y || a.mix.y) {
        float y[PC][V];
#pragma unroll
        for (int i = 0; i < PC; ++i)
#pragma unroll
            for (int v = 0; v < V; ++v) y[i][v] = 0.0f;
        if (a.y) {
#pragma unroll(PC == 1 ? 4 : 1)
            for (int z = 0; z < a.ysplit; ++z) {
                const float* yr = a.y + (long)z * a.ystride + (long)row * D;
#pragma unroll
                for (int i = 0; i < PC; ++i) {
                    float q[V];
                    ldv(yr + dd[i], q);
#pragma unroll
                    for (int v = 0; v < V; ++v) y[i][v] += q[v];
                }
            }
        }
        if (a.mix.y) {
            const ExpertMix& m = a.mix;
            if (m.gate) {
                const float g = m.gate[row];
#pragma unroll
                for (int i = 0; i < PC; ++i)
#pragma unroll
                    for (int v = 0; v < V; ++v) y[i][v] *= g;
            }
            const T* hr = reinterpret_cast<const T*>(m.h) + (long)row * m.ldh;
            const long e0 = (long)row * m.top;
            // every entry's row is read and dropped where an identity was chosen (it holds nothing then): no load waits
            // for the choice; KB rows in flight together
            constexpr int KB = PC == 1 ? 8 : 1;
            float self = 0.0f;
            for (int k0 = 0; k0 < m.top; k0 += KB) {
                float q[KB][PC][V];
#pragma unroll
                for (int j = 0; j < KB; ++j)
#pragma unroll
                    for (int i = 0; i < PC; ++i)
                        ldv(reinterpret_cast<const T*>(m.y) + (e0 + min(k0 + j, m.top - 1)) * m.ldy + dd[i], q[j][i]);
#pragma unroll
                for (int j = 0; j < KB; ++j) {
                    const long e = e0 + min(k0 + j, m.top - 1);
                    const float w = k0 + j < m.top ? m.w[e] : 0.0f;
                    const bool real = m.sel[e] < m.experts && k0 + j < m.top;
                    self += real ? 0.0f : w;
#pragma unroll
                    for (int i = 0; i < PC; ++i)
#pragma unroll
                        for (int v = 0; v < V; ++v) y[i][v] = real ? fmaf(w, q[j][i][v], y[i][v]) : y[i][v];
                }
            }
#pragma unroll
            for (int i = 0; i < PC; ++i) {
                float q[V];
                ldv(hr + dd[i], q);
#pragma unroll
                for (int v = 0; v < V; ++v) y[i][v] = fmaf(self, q[v], y[i][v]);
            }
        }
#pragma unroll
        for (int i = 0; i < PC; ++i)
#pragma unroll
            for (int v = 0; v < V; ++v) x[i][v] = fmaf(a.mult, y[i][v], x[i][v]);
    }
    rload(tid >> 6, 0);  // in flight during the norm (loads return in order: not ahead of the update's)
    const float corr = RT ? bf2f(rt.r.correction[min(tid & 63, rt.r.n - 1)]) : 0.0f;
    float ss = 0.0f;
#pragma unroll
    for (int i = 0; i < PC; ++i) {
        if (!ok[i]) continue;
#pragma unroll
        for (int v = 0; v < V; ++v) ss = fmaf(x[i][v], x[i][v], ss);
        if (!a.rows_idx && (a.ids || a.y || a.mix.y)) stv(Xr + dd[i], x[i]);
        if (a.tap) stv(a.tap + (long)row * D + dd[i], x[i]);
    }
    if (!a.h && !a.inv) return;
    ss = wave_sum(ss);
    if ((tid & 63) == 0) red[tid >> 6] = ss;
    __syncthreads();
    ss = 0.0f;
    for (int w = 0; w < NT / 64; ++w) ss += red[w];
    const float inv = 1.0f / sqrtf(ss / (float)D + a.eps);
    if (a.inv && tid == 0) a.inv[row] = inv;
    if (!a.h) return;
    T* h = reinterpret_cast<T*>(a.h) + (long)blockIdx.x * a.ldh;
    T* hs = reinterpret_cast<T*>(rsm + (RT ? route_words(rt.r.n, rt.r.groups) : 0));
    const float g = a.w_scalar ? bf2f(a.w[0]) : 0.0f;
    float part = 0.0f;  // of the gate
#pragma unroll
    for (int i = 0; i < PC; ++i) {
        if (!ok[i]) continue;
        float n[V], o[V];
#pragma unroll
        for (int v = 0; v < V; ++v) o[v] = n[v] = x[i][v] * inv * (a.w_scalar ? g : bf2f(a.w[dd[i] + v]));
        if constexpr (KT > 0) {
#pragma unroll
            for (int v = 0; v < V; ++v) {
                o[v] = fmaf(wk[KT - 1][i][v], n[v], o[v]);
#pragma unroll
                for (int j = 0; j < KT - 1; ++j) o[v] = fmaf(wk[KT - 2 - j][i][v], back[j][i][v], o[v]);
            }
            if (KT > 1) stv(ring + (long)(pos % KT) * D + dd[i], n);
        } else if (a.taps > 0) {
            const uint16_t* cw = a.cw + (long)dd[i] * a.taps;
            for (int j = 0; j < a.taps && j <= pos; ++j) {
                float q[V];
                if (j > 0) {
                    ldv(ring + (long)((pos - j) % a.taps) * D + dd[i], q);
                } else {
#pragma unroll
                    for (int v = 0; v < V; ++v) q[v] = n[v];
                }
#pragma unroll
                for (int v = 0; v < V; ++v) o[v] = fmaf(bf2f(cw[v * a.taps + a.taps - 1 - j]), q[v], o[v]);
            }
            if (a.taps > 1) stv(ring + (long)(pos % a.taps) * D + dd[i], n);
        }
        stv(h + dd[i], o);
        if constexpr (RT) {
            stv(hs + dd[i], o);
#pragma unroll
            for (int v = 0; v < V; ++v) part = fmaf(gw[v], rbf(o[v]), part);
        }
    }
    for (int d = D + tid; d < a.ldh; d += NT) {
        stf(h + d, 0.0f);
        if constexpr (RT) stf(hs + d, 0.0f);
    }
    if constexpr (RT) {
        const RouteArgs& r = rt.r;
        const int lane = tid & 63, wave = tid >> 6;
        float* z = rsm;
        __shared__ float gate[16];
        part = wave_sum(part);
        if (lane == 0) gate[wave] = part;
        __syncthreads();
        for (int n0 = wave; n0 < rows_r; n0 += 16 * RR) {
            float acc[RR] = {};
            for (int k0 = 0; k0 < a.ldh; k0 += 512 * RK) {
                if (n0 > wave || k0 > 0) rload(n0, k0);
#pragma unroll
                for (int i = 0; i < RK; ++i) {
                    const int k = k0 + i * 512 + lane * 8;
                    const uint4 x = k < a.ldh ? *reinterpret_cast<const uint4*>(hs + k) : make_uint4(0, 0, 0, 0);
#pragma unroll
                    for (int q = 0; q < RR; ++q) acc[q] = dot8(rw[q][i], x, acc[q]);
                }
            }
#pragma unroll
            for (int q = 0; q < RR; ++q) acc[q] = wave_sum(acc[q]);
#pragma unroll
            for (int q = 0; q < RR; ++q)
                if (lane == 0 && n0 + 16 * q < rows_r) z[n0 + 16 * q] = acc[q];
        }
        __syncthreads();
        if (wave > 0) return;
        if (r.gate) {
            part = 0.0f;
#pragma unroll
            for (int w = 0; w < 16; ++w) part += gate[w];
            if (lane == 0) r.gate[row] = 1.0f / (1.0f + expf(-part));
        }
        const bool alone = a.rows == 1;  // nobody else counts: the used experts by place, -1 for an identity
        if (alone && lane == 0) r.active[0] = r.top;
        const auto correction = [&](int c) { return c < 64 ? corr : bf2f(r.correction[c]); };
        route_row(z, correction, r.n, r.groups, r.keep, r.top, lane, [&](int k, int e, float w) {
            const int at = row * r.top + k;
            r.sel[at] = e;
            r.w[at] = w;
            if (alone) {
                r.active[1 + k] = e < r.experts ? e : -1;
                if (e < r.experts) {
                    r.cnt[e] = 1;
                    r.list[(long)e * r.cap] = at;
                }
            } else if (e < r.experts) {
                const int m = atomicAdd(&r.cnt[e], 1);
                r.list[(long)e * r.cap + m] = at;
                if (m == 0) r.active[1 + atomicAdd(&r.active[0], 1)] = e;
            }
        });
    }
}

template <typename T>
void residual_t(hipStream_t s, const ResidualArgs& a) {
    auto go = [&](auto kern, int v) {
        const int threads = std::min(1024, (a.D / v + 63) / 64 * 64);
        hipLaunchKernelGGL(kern, dim3(a.rows), dim3(std::max(64, threads)), 0, s, a, RouterArgs{});
    };
    if (a.D % 4 == 0 && a.D <= 4096) {
        if (a.taps == 4) go(k_residual<T, 4, 1, false, 4>, 4);
        else if (a.taps == 3) go(k_residual<T, 4, 1, false, 3>, 4);
        else if (a.taps == 2) go(k_residual<T, 4, 1, false, 2>, 4);
        else go(k_residual<T, 4, 1, false, 0>, 4);
    } else if (a.D % 4 == 0) {
        go(k_residual<T, 4, 4, false, 0>, 4);
    } else if (a.D <= 1024) {
        go(k_residual<T, 1, 1, false, 0>, 1);
    } else {
        go(k_residual<T, 1, 16, false, 0>, 1);
    }
}

// ---------------------------------------------------------------- input convolution
// the norm's output at the sequence's relative row p (p < 0: an earlier step's, from the ring)
__device__ __forceinline__ float canon_at(const CanonArgs& a, const SeqInfo& q, int p, int c) {
    if (p >= 0) return a.X[(long)(q.off + p) * a.D + c] * a.inv[q.off + p] * bf2f(a.w[a.w_scalar ? 0 : c]);
    p += q.start;
    return p >= 0 ? a.ring[((long)q.slot * a.taps + p % a.taps) * a.D + c] : 0.0f;
}

// four channels per lane, KT taps in registers, each wave a run of consecutive rows
template <typename T, int KT>
__global__ void __launch_bounds__(256) k_canon(CanonArgs a) {
    const ChunkInfo ck = a.chunks[blockIdx.y];
    const SeqInfo q = a.seqs[ck.seq];
    const int lane = threadIdx.x & 63, wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
    const int run = (ck.len + 3) / 4, r0 = wave * run, r1 = min(ck.len, r0 + run);
    const int c = (blockIdx.x * 64 + lane) * 4;
    if (c >= a.D || r0 >= r1) return;
    float wk[KT][4], g[4], win[KT][4];
#pragma unroll
    for (int v = 0; v < 4; ++v) {
        g[v] = bf2f(a.w[a.w_scalar ? 0 : c + v]);
#pragma unroll
        for (int t = 0; t < KT; ++t) wk[t][v] = bf2f(a.cw[(long)(c + v) * KT + t]);
    }
    auto take = [&](int row, float (&n)[4]) {
        const float inv = a.inv[row];
        ld4(a.X + (long)row * a.D + c, n);
#pragma unroll
        for (int v = 0; v < 4; ++v) n[v] = n[v] * inv * g[v];
    };
#pragma unroll
    for (int t = 0; t < KT - 1; ++t) {
        const int p = ck.rel + r0 - (KT - 1) + t;
        if (p >= 0) {
            take(q.off + p, win[t]);
        } else {
#pragma unroll
            for (int v = 0; v < 4; ++v) win[t][v] = canon_at(a, q, p, c + v);
        }
    }
    T* h = reinterpret_cast<T*>(a.h);
#pragma unroll 4
    for (int r = r0; r < r1; ++r) {
        take(ck.row + r, win[KT - 1]);
        float y[4];
#pragma unroll
        for (int v = 0; v < 4; ++v) {
            y[v] = win[KT - 1][v];
#pragma unroll
            for (int t = KT - 1; t >= 0; --t) y[v] = fmaf(wk[t][v], win[t][v], y[v]);
#pragma unroll
            for (int t = 0; t + 1 < KT; ++t) win[t][v] = win[t + 1][v];
        }
        st4(h + (long)(ck.row + r) * a.ldh + c, y);
        if (c + 4 == a.D)
            for (int d = a.D; d < a.ldh; ++d) stf(h + (long)(ck.row + r) * a.ldh + d, 0.0f);
    }
}

// any number of taps and channels
template <typename T>
__global__ void __launch_bounds__(256) k_canon_any(CanonArgs a) {
    const ChunkInfo ck = a.chunks[blockIdx.y];
    const SeqInfo q = a.seqs[ck.seq];
    const int c = blockIdx.x * 64 + (threadIdx.x & 63);
    if (c >= a.ldh) return;
    T* h = reinterpret_cast<T*>(a.h);
    for (int r = threadIdx.x >> 6; r < ck.len; r += 4) {
        float y = 0.0f;
        if (c < a.D) {
            y = canon_at(a, q, ck.rel + r, c);
            for (int t = a.taps - 1; t >= 0; --t)
                y = fmaf(bf2f(a.cw[(long)c * a.taps + t]), canon_at(a, q, ck.rel + r - (a.taps - 1) + t, c), y);
        }
        stf(h + (long)(ck.row + r) * a.ldh + c, y);
    }
}

// the sequences' last taps - 1 rows of this step into the ring
__global__ void __launch_bounds__(256) k_canon_keep(CanonArgs a) {
    const int n = a.taps - 1;
    const SeqInfo q = a.seqs[blockIdx.y / n];
    const int c = blockIdx.x * 256 + threadIdx.x, p = q.len - 1 - (int)(blockIdx.y % n);
    if (c >= a.D || p < 0) return;
    a.ring[((long)q.slot * a.taps + (q.start + p) % a.taps) * a.D + c] = canon_at(a, q, p, c);
}

template <typename T>
void canon_t(hipStream_t s, const CanonArgs& a) {
    const dim3 grid((a.D + 255) / 256, a.nchunk);
    if (a.D % 4 == 0 && a.taps == 4) hipLaunchKernelGGL((k_canon<T, 4>), grid, dim3(256), 0, s, a);
    else if (a.D % 4 == 0 && a.taps == 3) hipLaunchKernelGGL((k_canon<T, 3>), grid, dim3(256), 0, s, a);
    else if (a.D % 4 == 0 && a.taps == 2) hipLaunchKernelGGL((k_canon<T, 2>), grid, dim3(256), 0, s, a);
    else hipLaunchKernelGGL((k_canon_any<T>), dim3((a.ldh + 63) / 64, a.nchunk), dim3(256), 0, s, a);
    if (a.taps > 1)
        hipLaunchKernelGGL(k_canon_keep, dim3((a.D + 255) / 256, a.nseq * (a.taps - 1)), dim3(256), 0, s, a);
}

}  // namespace

void residual_norm(hipStream_t s, Act act, const ResidualArgs& a) {
    if (a.rows <= 0) return;
    if (act == ACT_F32) residual_t<float>(s, a);
    else residual_t<uint16_t>(s, a);
}

bool residual_route_fits(Act act, int rows, int D) {
    return act == ACT_BF16 && rows <= kRouteRows && D % 4 == 0 && D <= 4096;
}

void residual_route(hipStream_t s, const ResidualArgs& a, const uint16_t* W, int ldw, const RouteArgs& r) {
    const size_t lds = (size_t)route_words(r.n, r.groups) * sizeof(float) + (size_t)a.ldh * sizeof(uint16_t);
    hipLaunchKernelGGL((k_residual<uint16_t, 4, 1, true, 0>), dim3(a.rows), dim3(1024), lds, s, a, RouterArgs{W, ldw, r});
}

void canon(hipStream_t s, Act act, const CanonArgs& a) {
    if (act == ACT_F32) canon_t<float>(s, a);
    else canon_t<uint16_t>(s, a);
}

}  // namespace pgmi
