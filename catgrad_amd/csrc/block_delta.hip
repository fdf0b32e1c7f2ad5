// Gated delta rule with a decay per key channel (cg_block_channel_delta).
//
//   delta_conv_kernel      a workgroup per token: the short convolutions with silu, unit q and k, decay and step size of
//                          every head, and the convolutions' next state
//   delta_scan_kernel      the recurrence: a wave owns four columns of a head's state, its lanes the rows
//   delta_finish_kernel    a wave per (token, head): the norm over the head's values and the gate
#include "blocks.hpp"
#include "device_utils.hpp"

#include <algorithm>

namespace cg {
namespace {

constexpr int kThreads = 256, kWaves = 4;

__device__ __forceinline__ float wave_sum(float v) {
#pragma unroll
    for (int d = 32; d > 0; d >>= 1) v += __shfl_xor(v, d, 64);
    return v;
}
// sum over the 16 lanes of a row of lanes, for each of them
__device__ __forceinline__ float row16_sum(float v) {
    v += __int_as_float(__builtin_amdgcn_update_dpp(0, __float_as_int(v), 0x128, 0xF, 0xF, false)); // row_ror:8
    v += __int_as_float(__builtin_amdgcn_update_dpp(0, __float_as_int(v), 0x124, 0xF, 0xF, false)); // row_ror:4
    v += __int_as_float(__builtin_amdgcn_update_dpp(0, __float_as_int(v), 0x122, 0xF, 0xF, false)); // row_ror:2
    v += __int_as_float(__builtin_amdgcn_update_dpp(0, __float_as_int(v), 0x121, 0xF, 0xF, false)); // row_ror:1
    return v;
}
__device__ __forceinline__ float sigmoid(float z) { return 1.0f / (1.0f + expf(-z)); }
__device__ __forceinline__ float softplus(float z) { return z > 20.0f ? z : log1pf(expf(z)); }

// What the scan reads, per token: unit queries (times dim^-1/2) and keys [G * dim], values [H * vdim], the logarithms of
// the decays [H * dim], step sizes [H].
struct DeltaInputs {
    float *q, *k, *v, *log_g, *beta;
};

// Channel c of the three projections side by side, at time t of sequence b (t < 0: what the state kept).
__device__ __forceinline__ float conv_input(const DeltaPlan &p, uint32_t b, int t, uint32_t c) {
    const uint32_t kc = p.kv_heads * p.dim, vc = p.heads * p.vdim;
    if (t < 0) return p.conv_state ? p.conv_state[((int64_t)b * (p.taps - 1) + (t + (int)p.taps - 1)) * (2 * kc + vc) + c] : 0.0f;
    const int64_t r = (int64_t)b * p.S + t;
    return c < kc ? p.q.p[r * p.q.pitch + c] : c < 2 * kc ? p.k.p[r * p.k.pitch + c - kc] : p.v.p[r * p.v.pitch + c - 2 * kc];
}
__device__ __forceinline__ float conv_silu(const DeltaPlan &p, uint32_t b, int t, uint32_t c) {
    const uint32_t kc = p.kv_heads * p.dim;
    const float *w = c < kc ? p.conv_q + (int64_t)c * p.taps : c < 2 * kc ? p.conv_k + (int64_t)(c - kc) * p.taps : p.conv_v + (int64_t)(c - 2 * kc) * p.taps;
    float s = 0.0f;
    for (uint32_t i = 0; i < p.taps; i++) s = fmaf(conv_input(p, b, t - (int)(p.taps - 1 - i), c), w[i], s);
    return s * sigmoid(s);
}

__global__ __launch_bounds__(kThreads) void delta_conv_kernel(const DeltaPlan p, const DeltaInputs o, const float *__restrict__ decay) {
    const uint32_t r = blockIdx.x, b = r / p.S, t = r - b * p.S, wave = threadIdx.x >> 6, lane = threadIdx.x & 63;
    const uint32_t kc = p.kv_heads * p.dim, vc = p.heads * p.vdim, C = 2 * kc + vc, past = p.taps - 1;
    for (uint32_t u = wave; u < 2 * p.kv_heads; u += kWaves) { // q heads, then k heads
        const uint32_t c0 = u * p.dim;
        float v[4], ss = 0.0f; // (dim <= 256)
#pragma unroll
        for (int i = 0; i < 4; i++) {
            const uint32_t d = lane + 64 * i;
            v[i] = d < p.dim ? conv_silu(p, b, (int)t, c0 + d) : 0.0f;
            ss = fmaf(v[i], v[i], ss);
        }
        float f = 1.0f / sqrtf(wave_sum(ss) + 1e-6f);
        if (u < p.kv_heads) f *= 1.0f / sqrtf((float)p.dim);
        float *dst = u < p.kv_heads ? o.q + (int64_t)r * kc + c0 : o.k + (int64_t)r * kc + (c0 - kc);
#pragma unroll
        for (int i = 0; i < 4; i++) {
            const uint32_t d = lane + 64 * i;
            if (d < p.dim) dst[d] = v[i] * f;
        }
    }
    for (uint32_t c = threadIdx.x; c < vc; c += kThreads) o.v[(int64_t)r * vc + c] = conv_silu(p, b, (int)t, 2 * kc + c);
    const uint32_t hd = p.heads * p.dim;
    for (uint32_t i = threadIdx.x; i < hd; i += kThreads)
        o.log_g[(int64_t)r * hd + i] = -expf(p.a_log[i / p.dim]) * softplus(decay[(int64_t)r * hd + i] + p.dt_bias[i]);
    for (uint32_t h = threadIdx.x; h < p.heads; h += kThreads) o.beta[(int64_t)r * p.heads + h] = sigmoid(p.beta.p[(int64_t)r * p.beta.pitch + h]);
    // the last taps - 1 inputs, the ones this portion did not bring from the old state
    if (t == 0)
        for (uint32_t i = threadIdx.x; i < past * C; i += kThreads) {
            const uint32_t j = i / C, c = i - j * C;
            p.conv_out[((int64_t)b * past + j) * C + c] = conv_input(p, b, (int)(p.S + j) - (int)past, c);
        }
}

// Lane (l & 15) of four rows of lanes holds rows (l & 15) * R .. + R of one column of the state.
template <int R>
__global__ __launch_bounds__(kThreads) void delta_scan_kernel(const DeltaPlan p, const DeltaInputs in, float *__restrict__ out) {
    const uint32_t h = blockIdx.y, b = blockIdx.z, g = h / (p.heads / p.kv_heads), lane = threadIdx.x & 63;
    const uint32_t c = (blockIdx.x * kWaves + (threadIdx.x >> 6)) * 4 + (lane >> 4), d0 = (lane & 15) * R;
    const bool live = c < p.vdim;
    float S[R];
    const int64_t sb = (((int64_t)b * p.heads + h) * p.dim) * p.vdim;
#pragma unroll
    for (int i = 0; i < R; i++) S[i] = live && p.state && d0 + i < p.dim ? p.state[sb + (int64_t)(d0 + i) * p.vdim + c] : 0.0f;
    const uint32_t kc = p.kv_heads * p.dim, vc = p.heads * p.vdim, hd = p.heads * p.dim;
    const float *q = in.q + (int64_t)b * p.S * kc + g * p.dim, *k = in.k + (int64_t)b * p.S * kc + g * p.dim;
    const float *lg = in.log_g + (int64_t)b * p.S * hd + h * p.dim, *v = in.v + (int64_t)b * p.S * vc + h * p.vdim, *be = in.beta + (int64_t)b * p.S * p.heads + h;
    float *o = out + (int64_t)b * p.S * vc + h * p.vdim;
    float nq[R], nk[R], ng[R], nv = 0.0f, nb = 0.0f;
    auto ask = [&](uint32_t t) {
#pragma unroll
        for (int i = 0; i < R; i++) {
            const bool in_row = d0 + i < p.dim;
            nq[i] = in_row ? q[(int64_t)t * kc + d0 + i] : 0.0f;
            nk[i] = in_row ? k[(int64_t)t * kc + d0 + i] : 0.0f;
            ng[i] = in_row ? lg[(int64_t)t * hd + d0 + i] : 0.0f;
        }
        nv = live ? v[(int64_t)t * vc + c] : 0.0f;
        nb = be[(int64_t)t * p.heads];
    };
    ask(0);
    for (uint32_t t = 0; t < p.S; t++) {
        float cq[R], ck[R];
        const float cv = nv, cb = nb;
        float read = 0.0f;
#pragma unroll
        for (int i = 0; i < R; i++) {
            cq[i] = nq[i];
            ck[i] = nk[i];
            S[i] *= expf(ng[i]);
            read = fmaf(S[i], ck[i], read);
        }
        if (t + 1 < p.S) ask(t + 1);
        const float u = cb * (cv - row16_sum(read));
        float y = 0.0f;
#pragma unroll
        for (int i = 0; i < R; i++) {
            S[i] = fmaf(ck[i], u, S[i]);
            y = fmaf(S[i], cq[i], y);
        }
        y = row16_sum(y);
        if (live && (lane & 15) == 0) o[(int64_t)t * vc + c] = y;
    }
#pragma unroll
    for (int i = 0; i < R; i++)
        if (live && d0 + i < p.dim) p.state_out[sb + (int64_t)(d0 + i) * p.vdim + c] = S[i];
}

// gate: [B * S, heads * vdim]; in place on `o`
__global__ __launch_bounds__(kThreads) void delta_finish_kernel(const DeltaPlan p, const float *__restrict__ gate, float *__restrict__ o, const uint64_t heads_in_all) {
    const uint64_t w = (uint64_t)blockIdx.x * kWaves + (threadIdx.x >> 6);
    if (w >= heads_in_all) return;
    const uint32_t lane = threadIdx.x & 63;
    float *x = o + w * p.vdim;
    const float *gt = gate + w * p.vdim;
    float ss = 0.0f;
    for (uint32_t d = lane; d < p.vdim; d += 64) ss = fmaf(x[d], x[d], ss);
    const float f = 1.0f / sqrtf(wave_sum(ss) / (float)p.vdim + p.eps);
    for (uint32_t d = lane; d < p.vdim; d += 64) x[d] = x[d] * f * p.norm[d] * sigmoid(gt[d]);
}

int launched(const char *what) {
    const hipError_t e = hipGetLastError();
    return e == hipSuccess ? CG_OK : hip_fail(e, what);
}

struct Scratch {
    cg_backend *be;
    std::vector<std::pair<void *, size_t>> mem;
    explicit Scratch(cg_backend *b) : be(b) {}
    int get(size_t floats, float **p) {
        void *m;
        size_t cls;
        int rc = be->pool.alloc(floats * 4, &m, &cls);
        if (!rc) mem.emplace_back(m, cls);
        *p = static_cast<float *>(m);
        return rc;
    }
    ~Scratch() {
        for (auto &a : mem) be->pool.free(a.first, a.second);
    }
};

// x[rows, rank] . w^T [n, rank] in f32
int low_rank(cg_backend *be, const Rows &x, uint32_t rows, const float *w, uint32_t n, uint32_t rank, float *y) {
    if (few_rows_slots(rows, (uint64_t)staged_pitch(rank) * 4)) {
        ProductInput in;
        in.x = x;
        in.k1 = in.k = rank;
        Weight wt;
        wt.p = w;
        wt.pitch = rank;
        wt.n = n;
        wt.k = rank;
        return launch_few_rows_linear(be, in, rows, wt, nullptr, 1.0f, y);
    }
    Buffer bx, bw, bo; // borrowed memory
    cg_tensor tx, tw, to;
    auto view = [&](cg_tensor &t, Buffer &b, const void *p, int64_t d0, int64_t d1, int64_t s0, int64_t s1) {
        b.be = be;
        b.ptr = const_cast<void *>(p);
        t.be = be;
        t.buf = &b;
        t.rank = 2;
        t.dims[0] = d0;
        t.dims[1] = d1;
        t.strides[0] = s0;
        t.strides[1] = s1;
    };
    view(tx, bx, x.p, rows, rank, x.pitch, 1);
    view(tw, bw, w, rank, n, 1, rank);
    view(to, bo, y, rows, n, n, 1);
    const int rc = launch_matmul(be, &tx, &tw, &to);
    tx.buf = tw.buf = to.buf = nullptr;
    return rc;
}

} // namespace

int launch_channel_delta(cg_backend *be, const DeltaPlan &p) {
    const uint32_t rows = p.B * p.S, kc = p.kv_heads * p.dim, vc = p.heads * p.vdim, hd = p.heads * p.dim;
    Scratch mem(be);
    DeltaInputs in;
    float *decay, *gate;
    for (auto &m : {std::make_pair(&in.q, kc), std::make_pair(&in.k, kc), std::make_pair(&in.v, vc), std::make_pair(&in.log_g, hd),
                    std::make_pair(&in.beta, p.heads), std::make_pair(&decay, hd), std::make_pair(&gate, vc)})
        if (int rc = mem.get((size_t)rows * m.second, m.first)) return rc;
    if (int rc = low_rank(be, p.decay, rows, p.decay_w, hd, p.decay_rank, decay)) return rc;
    if (int rc = low_rank(be, p.gate, rows, p.gate_w, vc, p.gate_rank, gate)) return rc;
    hipLaunchKernelGGL(delta_conv_kernel, dim3(rows), dim3(kThreads), 0, be->stream, p, in, decay);
    {
        ProfScope prof(be, CG_K_RECURRENCE, (double)rows * p.heads * p.dim * p.vdim * 7.0);
        const dim3 grid((p.vdim + 4 * kWaves - 1) / (4 * kWaves), p.heads, p.B);
        const int r = (int)((p.dim + 15) / 16);
        if (r <= 1) hipLaunchKernelGGL((delta_scan_kernel<1>), grid, dim3(kThreads), 0, be->stream, p, in, p.out);
        else if (r <= 2) hipLaunchKernelGGL((delta_scan_kernel<2>), grid, dim3(kThreads), 0, be->stream, p, in, p.out);
        else if (r <= 4) hipLaunchKernelGGL((delta_scan_kernel<4>), grid, dim3(kThreads), 0, be->stream, p, in, p.out);
        else if (r <= 8) hipLaunchKernelGGL((delta_scan_kernel<8>), grid, dim3(kThreads), 0, be->stream, p, in, p.out);
        else hipLaunchKernelGGL((delta_scan_kernel<16>), grid, dim3(kThreads), 0, be->stream, p, in, p.out);
    }
    const uint64_t n = (uint64_t)rows * p.heads;
    hipLaunchKernelGGL(delta_finish_kernel, dim3((uint32_t)((n + kWaves - 1) / kWaves)), dim3(kThreads), 0, be->stream, p, gate, p.out, n);
    return launched("channel_delta");
}

} // namespace cg
