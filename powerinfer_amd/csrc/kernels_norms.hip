// Layers with a norm before and after every sublayer: norms in groups, the sum that closes a sublayer together with the norm in front of the next
// one, and the norm with a causal convolution over time behind it.
#include "layer_types.hpp"
#include "mixers.hpp"

namespace {

constexpr int kNormMaxCols = 32768;

// scale[r * groups + g] = 1 / root mean square of group g of row r, for `rows` rows (at(r): their first value, in global memory or LDS).  part:
// group_parts floats.  Every (row, group) falls into equal pieces so that all waves have one.
__host__ __device__ inline int group_parts(int rows, int groups, int waves) { const int n = rows * groups; return n >= waves ? n : (waves + n - 1) / n * n; }
template <typename AT>
__device__ void group_scales(float * part, float * scale, int rows, int groups, int cols, float eps, AT && at) {
    const int nw = blockDim.x >> 6, wave = threadIdx.x >> 6, lane = threadIdx.x & 63, size = cols / groups, n = rows * groups, segs = group_parts(rows, groups, nw) / n;
    const int seg = ((size + segs - 1) / segs + 3) / 4 * 4;
    const bool quads = (size & 3) == 0;
    for (int task = wave; task < n * segs; task += nw) {
        const int rg = task / segs, s = task % segs, r = rg / groups, lo = min(s * seg, size), hi = min(lo + seg, size);
        const float * p = at(r) + (rg % groups) * size;
        float sum = 0.0f;
        if (quads) {
#pragma unroll 4
            for (int c = lo + lane * 4; c < hi; c += 256) {
                const float4 v = *reinterpret_cast<const float4 *>(p + c);
                sum = fmaf(v.x, v.x, fmaf(v.y, v.y, fmaf(v.z, v.z, fmaf(v.w, v.w, sum))));
            }
        } else {
            for (int c = lo + lane; c < hi; c += 64) sum = fmaf(p[c], p[c], sum);
        }
        sum = pi_wave_sum(sum);
        if (lane == 0) part[task] = sum;
    }
    __syncthreads();
    for (int i = threadIdx.x; i < n; i += blockDim.x) {
        float s = 0.0f;
        for (int k = 0; k < segs; ++k) s += part[i * segs + k];
        scale[i] = pi_inv_sqrt(s / (float)size + eps);
    }
    __syncthreads();
}

// one token a workgroup, its row in LDS
template <typename ST>
__global__ void sum_norm_kernel(pi_sum_norm p) {
    extern __shared__ __align__(16) float sm[];
    const int t = blockIdx.x, tid = threadIdx.x, nt = blockDim.x, size = p.cols / p.groups;
    float * buf = sm, * scale = sm + (p.cols + 3) / 4 * 4, * part = scale + p.groups;
    const size_t base = (size_t)(p.rows ? p.rows[t] : t) * p.cols;
    const bool quads = (p.cols & 3) == 0 && (size & 3) == 0;      // four columns lie in one group
    if (p.w) {
        const float * mix = p.mix ? p.mix + base : nullptr;
        if (quads) {
            struct alignas(4 * sizeof(ST)) Quad { ST v[4]; };
            for (int c = tid * 4; c < p.cols; c += nt * 4) {
                float4 v = mix ? *reinterpret_cast<const float4 *>(mix + c) : make_float4(0, 0, 0, 0);
                if (!mix) for (int k = 0; k < p.top; ++k) {
                    const Quad q = *reinterpret_cast<const Quad *>((const ST *)p.y + (size_t)p.inv[t * p.top + k] * p.cols + c);
                    const float w = p.y_w ? p.y_w[t * p.top + k] : 1.0f;
                    v.x = fmaf(w, from_st(q.v[0]), v.x); v.y = fmaf(w, from_st(q.v[1]), v.y); v.z = fmaf(w, from_st(q.v[2]), v.z); v.w = fmaf(w, from_st(q.v[3]), v.w);
                }
                *reinterpret_cast<float4 *>(buf + c) = v;
            }
        } else {
            for (int c = tid; c < p.cols; c += nt) {
                float v = mix ? mix[c] : 0.0f;
                if (!mix) for (int k = 0; k < p.top; ++k) v = fmaf(p.y_w ? p.y_w[t * p.top + k] : 1.0f, from_st(((const ST *)p.y)[(size_t)p.inv[t * p.top + k] * p.cols + c]), v);
                buf[c] = v;
            }
        }
        __syncthreads();
        group_scales(part, scale, 1, p.groups, p.cols, p.eps, [&](int) { return buf; });
        float * x = p.x + base, * keep = p.keep ? p.keep + base : nullptr;
        if (quads) {
            for (int c = tid * 4; c < p.cols; c += nt * 4) {
                const float f = p.mult * scale[c / size];
                const float4 b = *reinterpret_cast<const float4 *>(buf + c), w = *reinterpret_cast<const float4 *>(p.w + c), o = *reinterpret_cast<const float4 *>(x + c);
                const float4 v = make_float4(fmaf(f * b.x, w.x, o.x), fmaf(f * b.y, w.y, o.y), fmaf(f * b.z, w.z, o.z), fmaf(f * b.w, w.w, o.w));
                *reinterpret_cast<float4 *>(x + c) = v;
                if (keep) *reinterpret_cast<float4 *>(keep + c) = v;
                *reinterpret_cast<float4 *>(buf + c) = v;
            }
        } else {
            for (int c = tid; c < p.cols; c += nt) {
                const float v = fmaf(p.mult * scale[c / size] * buf[c], p.w[c], x[c]);
                x[c] = v;
                if (keep) keep[c] = v;
                buf[c] = v;
            }
        }
    } else {
        for (int c = tid; c < p.cols; c += nt) buf[c] = p.x[base + c];
    }
    if (!p.h) return;
    __syncthreads();
    group_scales(part, scale, 1, p.groups, p.cols, p.eps, [&](int) { return buf; });
    ST * h = (ST *)p.h;
    auto at = [&](int c) -> size_t { return p.ol ? pi_ol_index(t, c) : (size_t)t * p.ld + c; };
    if (quads && (p.ld & 3) == 0) {                    // (four columns from a multiple of four on lie together in both layouts)
        for (int c = tid * 4; c < p.cols; c += nt * 4) {
            const float f = scale[c / size];
            const float4 b = *reinterpret_cast<const float4 *>(buf + c), w = *reinterpret_cast<const float4 *>(p.w_next + c);
            const float v[4] = {f * b.x * w.x, f * b.y * w.y, f * b.z * w.z, f * b.w * w.w};
            store4(h + at(c), v, true, 4);
        }
    } else {
        for (int c = tid; c < p.cols; c += nt) h[at(c)] = to_st<ST>(scale[c / size] * buf[c] * p.w_next[c]);
    }
}

// An item of consecutive tokens of one run a workgroup: first the groups' scales of every row the item touches, then column by column the normed
// inputs of those rows and their convolution.
__host__ __device__ inline int conv_rows(int tokens, int taps) { return tokens + 2 * taps; }
template <typename ST>
__global__ __launch_bounds__(256) void conv_norm_kernel(pi_conv_norm p, int max_rows) {
    extern __shared__ __align__(16) float sm[];
    const int4 a = reinterpret_cast<const int4 *>(p.items)[2 * blockIdx.x], b = reinterpret_cast<const int4 *>(p.items)[2 * blockIdx.x + 1];
    const int t0 = a.x, n = a.y, off = a.z, len = a.w, slot = b.x, back = p.taps - 1, size = p.cols / p.groups;
    const bool head = off == 0, fresh = b.y != 0;
    const int before = min(off, back), run0 = t0 - off;
    // rows t0 - before .. t0 + n - 1, then (first item of a run) the run's last inputs behind them
    const int n_a = n + before, tail = head ? max(n, len - back) : len, rows = n_a + (head ? len - tail : 0);
    if (rows > max_rows) return;                       // (the launcher's bound)
    float * scale = sm, * part = sm + max_rows * p.groups;
    auto row = [&](int r) { return p.x + (size_t)(r < n_a ? t0 - before + r : run0 + tail + (r - n_a)) * p.cols; };
    group_scales(part, scale, rows, p.groups, p.cols, p.eps, row);
    float * state = p.state ? p.state + slot * p.slot_ld : nullptr;
    ST * h = (ST *)p.h;
    for (int c = threadIdx.x; c < p.cols; c += 256) {
        const int g = c / size;
        const float w = p.w[c], * tw = p.taps_w + c;
        auto input = [&](int i) -> float {             // the normed input at place i of the item (negative: before it)
            const int r = i + before;
            if (r >= 0) return p.x[(size_t)(t0 + i) * p.cols + c] * scale[r * p.groups + g] * w;
            const int s = off + i + back;              // before the run: row of the state
            return head && !fresh && s >= 0 ? state[(size_t)s * p.cols + c] : 0.0f;
        };
        for (int i = 0; i < n; ++i) {
            const float own = input(i);
            float v = 0.0f;
            for (int j = 0; j < back; ++j) v = fmaf(tw[(size_t)j * p.cols], input(i - back + j), v);
            v = fmaf(tw[(size_t)back * p.cols], own, v) + own;
            h[p.ol ? pi_ol_index(t0 + i, c) : (size_t)(t0 + i) * p.ld + c] = to_st<ST>(v);
        }
        if (!head || back == 0) continue;
        for (int s = 0; s < back; ++s) {               // ascending: an old row is read before it is overwritten
            const int i = len - back + s;              // place in the run
            float v;
            if (i < 0) v = fresh ? 0.0f : state[(size_t)(s + len) * p.cols + c];
            else if (i < n) v = input(i);
            else v = p.x[(size_t)(run0 + i) * p.cols + c] * scale[(n_a + i - tail) * p.groups + g] * w;
            state[(size_t)s * p.cols + c] = v;
        }
    }
}

// The same, four columns a thread, for up to BACK inputs ahead of a token and N >= BACK tokens of an item: a thread's inputs lie in registers, all requested together.
template <typename ST, int BACK, int N>
__global__ __launch_bounds__(1024) void conv_norm_quads_kernel(pi_conv_norm p, int max_rows) {
    extern __shared__ __align__(16) float sm[];
    const int4 a = reinterpret_cast<const int4 *>(p.items)[2 * blockIdx.x], b = reinterpret_cast<const int4 *>(p.items)[2 * blockIdx.x + 1];
    const int t0 = a.x, n = min(a.y, N), off = a.z, len = a.w, slot = b.x, size = p.cols / p.groups;
    const bool head = off == 0, fresh = b.y != 0;
    const int before = min(off, BACK), run0 = t0 - off, n_a = n + before, tail = head ? max(n, len - BACK) : len, rows = n_a + (head ? len - tail : 0);
    if (rows > max_rows) return;                       // (the launcher's bound)
    float * scale = sm, * part = sm + max_rows * p.groups;
    group_scales(part, scale, rows, p.groups, p.cols, p.eps, [&](int r) { return p.x + (size_t)(r < n_a ? t0 - before + r : run0 + tail + (r - n_a)) * p.cols; });
    float * state = p.state ? p.state + slot * p.slot_ld : nullptr;
    ST * h = (ST *)p.h;
    for (int c = threadIdx.x * 4; c < p.cols; c += blockDim.x * 4) {
        const int g = c / size;
        const auto quad = [&](const float * q) { return *reinterpret_cast<const float4 *>(q + c); };
        float4 u[BACK + N], tw[BACK + 1];              // inputs: place k - BACK of the item
        const float4 w = quad(p.w);
#pragma unroll
        for (int j = 0; j <= BACK; ++j) tw[j] = quad(p.taps_w + (size_t)j * p.cols);
#pragma unroll
        for (int k = 0; k < BACK + N; ++k) {
            const int i = k - BACK;
            u[k] = make_float4(0, 0, 0, 0);
            if (i >= n) continue;
            if (i + before >= 0) u[k] = quad(p.x + (size_t)(t0 + i) * p.cols);
            else if (head && !fresh) u[k] = quad(state + (size_t)k * p.cols);
        }
#pragma unroll
        for (int k = 0; k < BACK + N; ++k) {
            const int r = k - BACK + before;
            if (r < 0 || r >= n_a) continue;
            const float f = scale[r * p.groups + g];
            u[k] = make_float4(u[k].x * f * w.x, u[k].y * f * w.y, u[k].z * f * w.z, u[k].w * f * w.w);
        }
#pragma unroll
        for (int i = 0; i < N; ++i) {
            if (i >= n) break;
            float4 v = u[BACK + i];
#pragma unroll
            for (int j = 0; j <= BACK; ++j) {
                const float4 q = u[i + j];
                v = make_float4(fmaf(tw[j].x, q.x, v.x), fmaf(tw[j].y, q.y, v.y), fmaf(tw[j].z, q.z, v.z), fmaf(tw[j].w, q.w, v.w));
            }
            const float o[4] = {v.x, v.y, v.z, v.w};
            store4(h + (p.ol ? pi_ol_index(t0 + i, c) : (size_t)(t0 + i) * p.ld + c), o, true, 4);
        }
        if (!head || BACK == 0) continue;
#pragma unroll
        for (int s = 0; s < BACK; ++s) {
            const int i = len - BACK + s;              // place in the run
            float4 v = make_float4(0, 0, 0, 0);
            if (i >= n) {
                const float f = scale[(n_a + i - tail) * p.groups + g];
                const float4 q = quad(p.x + (size_t)(run0 + i) * p.cols);
                v = make_float4(q.x * f * w.x, q.y * f * w.y, q.z * f * w.z, q.w * f * w.w);
            } else {
#pragma unroll
                for (int k = 0; k < BACK + N; ++k) if (k == BACK + i) v = u[k];
            }
            *reinterpret_cast<float4 *>(state + (size_t)s * p.cols + c) = v;
        }
    }
}
template <typename ST> bool launch_conv_quads(const pi_conv_norm & p, int rows, size_t lds, hipStream_t st) {
    if ((p.cols / p.groups) % 4 || p.ld % 4 || p.slot_ld % 4 || p.taps > 5) return false;
    const dim3 grid(p.n_items), block(p.cols > 2048 ? 1024 : p.cols > 1024 ? 512 : 256);
    switch (p.taps) {
        case 1: hipLaunchKernelGGL((conv_norm_quads_kernel<ST, 0, 4>), grid, block, lds, st, p, rows); break;
        case 2: hipLaunchKernelGGL((conv_norm_quads_kernel<ST, 1, 4>), grid, block, lds, st, p, rows); break;
        case 3: hipLaunchKernelGGL((conv_norm_quads_kernel<ST, 2, 4>), grid, block, lds, st, p, rows); break;
        case 4: hipLaunchKernelGGL((conv_norm_quads_kernel<ST, 3, 4>), grid, block, lds, st, p, rows); break;
        default: hipLaunchKernelGGL((conv_norm_quads_kernel<ST, 4, 4>), grid, block, lds, st, p, rows);
    }
    return true;
}

}  // namespace

extern "C" {

int pi_k_sum_norm(int type, const pi_sum_norm * p, pi_stream_t stream) {
    if (!p || !p->x || p->T <= 0 || p->cols <= 0 || p->groups <= 0 || p->cols % p->groups || (p->w && (p->rows || !p->mix == !p->y || (p->y && (!p->inv || p->top <= 0)))) || (!p->w && !p->h) ||
        (p->h && (!p->w_next || p->ld < p->cols)))
        return pi::fail(PI_E_ARG, "pi_k_sum_norm: bad arguments");
    if (p->cols > kNormMaxCols || p->groups > 1024) return pi::fail(PI_E_UNSUPPORTED, "pi_k_sum_norm: up to 32768 columns in up to 1024 groups");
    if (p->h && p->ol && (type != PI_TYPE_BF16 || p->T > kBtMaxT || p->ld % 8)) return pi::fail(PI_E_ARG, "pi_k_sum_norm: operand layout needs BF16, T <= 16, ld % 8 == 0");
    const int block = p->cols > 2048 ? 1024 : p->cols > 1024 ? 512 : 256;
    const size_t lds = sizeof(float) * ((size_t)(p->cols + 3) / 4 * 4 + p->groups + group_parts(1, p->groups, block / 64));
    static bool raised = false;
    if (!raised) {
        PI_HIP_TRY(hipFuncSetAttribute(reinterpret_cast<const void *>(&sum_norm_kernel<bf16>), hipFuncAttributeMaxDynamicSharedMemorySize, 150 * 1024));
        PI_HIP_TRY(hipFuncSetAttribute(reinterpret_cast<const void *>(&sum_norm_kernel<float>), hipFuncAttributeMaxDynamicSharedMemorySize, 150 * 1024));
        raised = true;
    }
    if (type == PI_TYPE_BF16) hipLaunchKernelGGL(sum_norm_kernel<bf16>, dim3(p->T), dim3(block), lds, (hipStream_t)stream, *p);
    else if (type == PI_TYPE_F32) hipLaunchKernelGGL(sum_norm_kernel<float>, dim3(p->T), dim3(block), lds, (hipStream_t)stream, *p);
    else return pi::fail(PI_E_UNSUPPORTED, "pi_k_sum_norm: type");
    return pi::check_launch("pi_k_sum_norm");
}

int pi_k_conv_tokens(int T, int taps) { return T <= 16 ? (taps > 2 ? taps - 1 : 1) : taps > 5 ? taps - 1 : 4; }

int pi_k_conv_norm(int type, const pi_conv_norm * p, pi_stream_t stream) {
    if (!p || !p->x || !p->w || !p->taps_w || !p->items || !p->h || p->T <= 0 || p->n_items <= 0 || p->cols <= 0 || p->groups <= 0 || p->cols % p->groups || p->taps <= 0 || p->ld < p->cols ||
        (p->taps > 1 && (!p->state || p->slot_ld < (size_t)(p->taps - 1) * p->cols)))
        return pi::fail(PI_E_ARG, "pi_k_conv_norm: bad arguments");
    if (p->ol && (type != PI_TYPE_BF16 || p->T > kBtMaxT || p->ld % 8)) return pi::fail(PI_E_ARG, "pi_k_conv_norm: operand layout needs BF16, T <= 16, ld % 8 == 0");
    const int rows = conv_rows(pi_k_conv_tokens(p->T, p->taps), p->taps);
    const size_t lds = sizeof(float) * ((size_t)rows * p->groups + group_parts(rows, p->groups, 16) + 16);
    if (lds > 64 * 1024) return pi::fail(PI_E_UNSUPPORTED, "pi_k_conv_norm: taps x groups");
    if (type != PI_TYPE_BF16 && type != PI_TYPE_F32) return pi::fail(PI_E_UNSUPPORTED, "pi_k_conv_norm: type");
    hipStream_t st = (hipStream_t)stream;
    if (type == PI_TYPE_BF16 ? launch_conv_quads<bf16>(*p, rows, lds, st) : launch_conv_quads<float>(*p, rows, lds, st)) return pi::check_launch("pi_k_conv_norm");
    if (type == PI_TYPE_BF16) hipLaunchKernelGGL(conv_norm_kernel<bf16>, dim3(p->n_items), dim3(256), lds, st, *p, rows);
    else hipLaunchKernelGGL(conv_norm_kernel<float>, dim3(p->n_items), dim3(256), lds, st, *p, rows);
    return pi::check_launch("pi_k_conv_norm");
}

}  // extern "C"
