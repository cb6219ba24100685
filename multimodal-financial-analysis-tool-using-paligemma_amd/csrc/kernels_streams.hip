// kernels_streams.hip -- residual streams (hyper-connections) with the grouped RMS norm of the next sublayer:
// one pass over a row's streams updates them from the finished sublayer's output, reads the next sublayer's
// input and normalises it.  Streams, sums and norms are fp32.
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

template <typename T, int SM>
void launch(hipStream_t s, const StreamsArgs& a) {
    const size_t lds = (size_t)(a.D + NT / 64 + a.groups) * sizeof(float);
    auto go = [&](auto kern) {
        if (lds > 64 * 1024)
            (void)hipFuncSetAttribute(reinterpret_cast<const void*>(kern), hipFuncAttributeMaxDynamicSharedMemorySize,
                                      (int)lds);
        hipLaunchKernelGGL(kern, dim3(a.rows), dim3(NT), lds, s, a);
    };
    if (a.D % 4 == 0) go(k_streams<T, SM, 4>);
    else go(k_streams<T, SM, 1>);
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
