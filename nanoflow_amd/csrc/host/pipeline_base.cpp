// What every schedule shares: construction, and streams restricted to a set of compute units.
#include "pipeline.h"

PipelineBase::PipelineBase(vortexInitData* input_data, int nrank, int nranks, int vnranks)
    : input_data(input_data),
      rank(nrank),
      nranks(nranks),
      vnranks(vnranks),
      tmpBufferM(input_data->tmp_buffer, input_data->tmp_buffer_size) {
  tensorlog::configure();  // NANOFLOW_TENSOR_LOG is read when a pipeline is created
}

// CUs first_cu .. first_cu + num_cus - 1 in the numbering of the CU mask, whose bit i is a CU of XCD
// i % 8 on this part: a range of 8 n bits is n CUs of every XCD, so both streams of a split keep
// all eight L2s and memory ports.
hipStream_t createPipelineStream(int first_cu, int num_cus) {
  hipStream_t s = nullptr;
  if (num_cus <= 0) {
    HIP_CHECK(hipStreamCreateWithFlags(&s, hipStreamNonBlocking));
    return s;
  }
  hipDeviceProp_t prop;
  int dev = 0;
  HIP_CHECK(hipGetDevice(&dev));
  HIP_CHECK(hipGetDeviceProperties(&prop, dev));
  const int total = prop.multiProcessorCount;
  const int words = (total + 31) / 32;
  std::vector<uint32_t> mask(words, 0u);
  for (int cu = first_cu; cu < first_cu + num_cus && cu < total; ++cu) mask[cu / 32] |= 1u << (cu % 32);
  HIP_CHECK(hipExtStreamCreateWithCUMask(&s, (uint32_t)words, mask.data()));
  return s;
}
