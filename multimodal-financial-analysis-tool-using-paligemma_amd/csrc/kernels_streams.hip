// kernels_streams.hip -- residual streams (hyper-connections) with the grouped RMS norm of the next sublayer:
// one pass over a row's streams updates them from the finished sublayer's output, reads the next sublayer's
// input and normalises it.  Streams, sums and norms are fp32.
#include <algorithm>

#include "act.h"
#include "decoder.h"

namespace pgmi {

namespace {

constexpr int NT = 256;

// One workgroup per row.  SM: compile-time bound on the streams held in registers (S <= SM).
// V: elements per access (4 when D % 4 == 0, else 1).
template <typename T, int SM, int V>
__global__ void __launch_bounds__(NT) k_streams(StreamsArgs a) {
    extern __shared__ float u_[];  // [D] then [64] reduction words, then [groups]
    float* red = u_ + a.D;
    float* inv = red + NT / 64;
    __shared__ float cin[SM], cout[SM], cmix[SM * SM];
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
    const int S = a.S, D = a.D;
    const int row = a.rows_idx ? a.rows_idx[blockIdx.x] : blockIdx.x;
    if (tid < SM) {
        cin[tid] = tid < S ? (a.in ? bf2f(a.in[tid]) : 1.0f) : 0.0f;
        cout[tid] = tid < S && a.out ? bf2f(a.out[tid]) : 0.0f;
    }
    for (int i = tid; i < SM * SM; i += NT) {
        const int f = i / SM, t = i % SM;
        cmix[i] = (f < S && t < S) ? (a.mix ? bf2f(a.mix[f * S + t]) : (f == t ? 1.0f : 0.0f)) : 0.0f;
    }
    __syncthreads();
    float* Xr = a.X + (long)row * S * D;
    const uint16_t* er = nullptr;
    if (a.ids) {
        long id = a.ids[row];
        id = id < 0 ? 0 : (id >= a.vocab ? a.vocab - 1 : id);
        er = a.E + id * D;
    }
    for (int d = tid * V; d < D; d += NT * V) {
        float x[SM][V];
        if (er) {
#pragma unroll
            for (int v = 0; v < V; ++v) {
                const float e = bf2f(er[d + v]) * a.escale;
#pragma unroll
                for (int s = 0; s < SM; ++s) x[s][v] = s < S ? e : 0.0f;
            }
        } else {
            float o[SM][V], y[V];
#pragma unroll
            for (int s = 0; s < SM; ++s) {
                if (s < S) {
                    if constexpr (V == 4) {
                        const float4 q = *reinterpret_cast<const float4*>(Xr + (long)s * D + d);
                        o[s][0] = q.x; o[s][1] = q.y; o[s][2] = q.z; o[s][3] = q.w;
                    } else {
                        o[s][0] = Xr[(long)s * D + d];
                    }
                } else {
#pragma unroll
                    for (int v = 0; v < V; ++v) o[s][v] = 0.0f;
                }
            }
#pragma unroll
            for (int v = 0; v < V; ++v) y[v] = 0.0f;
            for (int z = 0; z < a.ysplit; ++z) {
                const float* yr = a.y + (long)z * a.ystride + (long)row * D + d;
                if constexpr (V == 4) {
                    const float4 q = *reinterpret_cast<const float4*>(yr);
                    y[0] += q.x; y[1] += q.y; y[2] += q.z; y[3] += q.w;
                } else {
                    y[0] += yr[0];
                }
            }
#pragma unroll
            for (int t = 0; t < SM; ++t)
#pragma unroll
                for (int v = 0; v < V; ++v) {
                    float acc = cout[t] * y[v];
#pragma unroll
                    for (int s = 0; s < SM; ++s) acc = fmaf(cmix[s * SM + t], o[s][v], acc);
                    x[t][v] = acc;
                }
        }
        float u[V], sum[V];
#pragma unroll
        for (int v = 0; v < V; ++v) {
            u[v] = 0.0f;
            sum[v] = 0.0f;
#pragma unroll
            for (int s = 0; s < SM; ++s) {
                u[v] = fmaf(cin[s], x[s][v], u[v]);
                sum[v] += x[s][v];
            }
            u_[d + v] = u[v];
        }
        if (!a.rows_idx) {
#pragma unroll
            for (int s = 0; s < SM; ++s)
                if (s < S) {
                    if constexpr (V == 4)
                        *reinterpret_cast<float4*>(Xr + (long)s * D + d) = make_float4(x[s][0], x[s][1], x[s][2], x[s][3]);
                    else
                        Xr[(long)s * D + d] = x[s][0];
                }
        }
        if (a.tap) {
#pragma unroll
            for (int v = 0; v < V; ++v) a.tap[(long)row * D + d + v] = sum[v];
        }
    }
    if (!a.h) return;
    __syncthreads();
    const int P = D / a.groups;
    if (a.groups >= NT / 64) {  // a wave per group
        for (int g = wave; g < a.groups; g += NT / 64) {
            float q = 0.0f;
            for (int i = lane; i < P; i += 64) q = fmaf(u_[g * P + i], u_[g * P + i], q);
            q = wave_sum(q);
            if (lane == 0) inv[g] = 1.0f / sqrtf(q / (float)P + a.eps);
        }
        __syncthreads();
    } else {
        for (int g = 0; g < a.groups; ++g) {
            float q = 0.0f;
            for (int i = tid; i < P; i += NT) q = fmaf(u_[g * P + i], u_[g * P + i], q);
            q = wave_sum(q);
            if (lane == 0) red[wave] = q;
            __syncthreads();
            if (tid == 0) {
                float t = 0.0f;
                for (int w = 0; w < NT / 64; ++w) t += red[w];
                inv[g] = 1.0f / sqrtf(t / (float)P + a.eps);
            }
            __syncthreads();
        }
    }
    T* h = reinterpret_cast<T*>(a.h) + (long)blockIdx.x * a.ldh;
    for (int d = tid; d < a.ldh; d += NT) stf(h + d, d < D ? u_[d] * inv[d / P] * bf2f(a.w[d]) : 0.0f);
}

// The same for widths whose groups are whole numbers of 256 elements (D <= 8192): PC pieces of 4 elements per thread,
// every load of the row issued before the first is used, one barrier.
template <typename T, int SM, int PC>
__global__ void __launch_bounds__(1024) k_streams_v(StreamsArgs a) {
    __shared__ float red[32];
    const int tid = threadIdx.x, lane = tid & 63, NTV = blockDim.x;
    const int S = a.S, D = a.D, P = D / a.groups;
    const int row = a.rows_idx ? a.rows_idx[blockIdx.x] : blockIdx.x;
    float* Xr = a.X + (long)row * S * D;
    float x[PC][SM][4], y[PC][4], u[PC][4];
    ushort4 nw[PC];
    const uint16_t* er = nullptr;
    if (a.ids) {
        long id = a.ids[row];
        id = id < 0 ? 0 : (id >= a.vocab ? a.vocab - 1 : id);
        er = a.E + id * D;
    }
#pragma unroll
    for (int i = 0; i < PC; ++i) {
        const int d = (i * NTV + tid) * 4;
        const bool ok = d < D;
        const int dd = ok ? d : 0;
        nw[i] = a.h ? *reinterpret_cast<const ushort4*>(a.w + dd) : make_ushort4(0, 0, 0, 0);
#pragma unroll
        for (int v = 0; v < 4; ++v) y[i][v] = 0.0f;
        if (er) {
            float e[4];
            ld4(er + dd, e);
#pragma unroll
            for (int s = 0; s < SM; ++s)
#pragma unroll
                for (int v = 0; v < 4; ++v) x[i][s][v] = ok && s < S ? e[v] * a.escale : 0.0f;
        } else {
#pragma unroll
            for (int s = 0; s < SM; ++s) {
                if (s < S) ld4(Xr + (long)s * D + dd, x[i][s]);
                else x[i][s][0] = x[i][s][1] = x[i][s][2] = x[i][s][3] = 0.0f;
            }
        }
    }
    if (!er && a.mix) {
#pragma unroll 4
        for (int z = 0; z < a.ysplit; ++z) {
#pragma unroll
            for (int i = 0; i < PC; ++i) {
                const int d = (i * NTV + tid) * 4;
                float q[4];
                ld4(a.y + (long)z * a.ystride + (long)row * D + (d < D ? d : 0), q);
#pragma unroll
                for (int v = 0; v < 4; ++v) y[i][v] += q[v];
            }
        }
        float m[SM][SM], o[SM];
#pragma unroll
        for (int t = 0; t < SM; ++t) {
            o[t] = t < S ? bf2f(a.out[t]) : 0.0f;
#pragma unroll
            for (int s = 0; s < SM; ++s) m[s][t] = s < S && t < S ? bf2f(a.mix[s * S + t]) : 0.0f;
        }
#pragma unroll
        for (int i = 0; i < PC; ++i)
#pragma unroll
            for (int v = 0; v < 4; ++v) {
                float n[SM];
#pragma unroll
                for (int t = 0; t < SM; ++t) {
                    n[t] = o[t] * y[i][v];
#pragma unroll
                    for (int s = 0; s < SM; ++s) n[t] = fmaf(m[s][t], x[i][s][v], n[t]);
                }
#pragma unroll
                for (int t = 0; t < SM; ++t) x[i][t][v] = n[t];
            }
    }
    float c[SM];
#pragma unroll
    for (int s = 0; s < SM; ++s) c[s] = s < S ? (a.in ? bf2f(a.in[s]) : 1.0f) : 0.0f;
#pragma unroll
    for (int i = 0; i < PC; ++i) {
        const int d = (i * NTV + tid) * 4;
        const bool ok = d < D;
        float ss = 0.0f, sum[4];
#pragma unroll
        for (int v = 0; v < 4; ++v) {
            u[i][v] = sum[v] = 0.0f;
#pragma unroll
            for (int s = 0; s < SM; ++s) {
                u[i][v] = fmaf(c[s], x[i][s][v], u[i][v]);
                sum[v] += x[i][s][v];
            }
            ss = fmaf(u[i][v], u[i][v], ss);
        }
        if (!a.rows_idx && (er || a.mix) && ok) {
#pragma unroll
            for (int s = 0; s < SM; ++s)
                if (s < S) st4(Xr + (long)s * D + d, x[i][s]);
        }
        if (a.tap && ok) st4(a.tap + (long)row * D + d, sum);
        ss = wave_sum(ss);  // a wave's 256 elements lie in one group
        if (lane == 0) red[(i * NTV + tid) / 64] = ss;
    }
    if (!a.h) return;
    __syncthreads();
    T* h = reinterpret_cast<T*>(a.h) + (long)blockIdx.x * a.ldh;
#pragma unroll
    for (int i = 0; i < PC; ++i) {
        const int d = (i * NTV + tid) * 4;
        if (d >= D) continue;
        const int p0 = d / P * (P / 256);
        float q = 0.0f;
        for (int t = 0; t < P / 256; ++t) q += red[p0 + t];
        const float f = 1.0f / sqrtf(q / (float)P + a.eps);
        const float v[4] = {u[i][0] * f * bf2f(nw[i].x), u[i][1] * f * bf2f(nw[i].y), u[i][2] * f * bf2f(nw[i].z),
                            u[i][3] * f * bf2f(nw[i].w)};
        st4(h + d, v);
    }
}

template <typename T, int SM>
void launch(hipStream_t s, const StreamsArgs& a) {
    const size_t lds = (size_t)(a.D + NT / 64 + a.groups) * sizeof(float);
    auto go = [&](auto kern) {
        if (lds > 60 * 1024)
            (void)hipFuncSetAttribute(reinterpret_cast<const void*>(kern), hipFuncAttributeMaxDynamicSharedMemorySize,
                                      (int)lds);
        hipLaunchKernelGGL(kern, dim3(a.rows), dim3(NT), lds, s, a);
    };
    if ((a.D / a.groups) % 256 == 0 && a.D <= 8192) {
        const int threads = std::min(1024, a.D / 4);
        if (a.D <= 4096) hipLaunchKernelGGL((k_streams_v<T, SM, 1>), dim3(a.rows), dim3(threads), 0, s, a);
        else hipLaunchKernelGGL((k_streams_v<T, SM, 2>), dim3(a.rows), dim3(threads), 0, s, a);
    } else if (a.D % 4 == 0) {
        go(k_streams<T, SM, 4>);
    } else {
        go(k_streams<T, SM, 1>);
    }
}

template <typename T>
void launch_s(hipStream_t s, const StreamsArgs& a) {
    if (a.S <= 1) launch<T, 1>(s, a);
    else if (a.S <= 2) launch<T, 2>(s, a);
    else if (a.S <= 4) launch<T, 4>(s, a);
    else launch<T, 8>(s, a);
}

}  // namespace

void streams_norm(hipStream_t s, Act act, const StreamsArgs& a) {
    if (a.rows <= 0) return;
    if (act == ACT_F32) launch_s<float>(s, a);
    else launch_s<uint16_t>(s, a);
}

}  // namespace pgmi
